// Gated delta rule: short causal convolutions, unit norms, decays, the recurrence over tokens, the gated head norm.
// Everything here is fp32.
#include "stack.h"
#include "delta_rows.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

// silu of the convolutions at NE channels for the tokens t0 .. t0 + TW - 1 of sequence b: y[token][channel], zeros past the
// end.  Up to four taps the inputs slide through registers, each read once; more taps are gathered token by token.
constexpr int TW = 8;        // tokens per wave
template <int NE>
__device__ __forceinline__ void conv_tokens(const DeltaRows &a, int b, int t0, const int (&ch)[NE], const int (&col)[NE], const bool (&in)[NE],
                                            float (&y)[TW][NE])
{
    const int T = a.r.T, nt = min(TW, T - t0), C = 2 * a.KV * a.dim + a.H * a.vdim;
    if (a.taps <= 4) {
        float f[NE][4], x[NE][TW + 3];
#pragma unroll
        for (int i = 0; i < TW + 3; i++) {
            const int tt = t0 - 3 + i, p = a.r.pos + tt;
#pragma unroll
            for (int e = 0; e < NE; e++) {
                float v = 0.f;
                if (in[e] && tt < T && p >= 0) {
                    if (tt >= 0) v = a.cin[(size_t)(b * T + tt) * a.ldc + col[e]];
                    else if (-tt < a.taps) v = a.conv[((size_t)b * a.taps + p % a.taps) * C + ch[e]];
                }
                x[e][i] = v;
            }
        }
#pragma unroll
        for (int e = 0; e < NE; e++)
#pragma unroll
            for (int i = 0; i < 4; i++) f[e][i] = in[e] && i >= 4 - a.taps ? a.filters[(size_t)ch[e] * a.taps + i - (4 - a.taps)] : 0.f;
#pragma unroll
        for (int i = 0; i < TW; i++)
#pragma unroll
            for (int e = 0; e < NE; e++)
                y[i][e] = silu(fmaf(f[e][3], x[e][i + 3], fmaf(f[e][2], x[e][i + 2], fmaf(f[e][1], x[e][i + 1], f[e][0] * x[e][i]))));
    } else {
#pragma unroll
        for (int i = 0; i < TW; i++)
#pragma unroll
            for (int e = 0; e < NE; e++) y[i][e] = in[e] && i < nt ? silu(conv_at(a, b * T + t0 + i, ch[e], col[e])) : 0.f;
    }
}

// One wave per (unit, TW tokens): units 0 .. KV-1 finish q and k of a key head, the others 64 channels of the values.  A
// lane holds channels lane, lane + 64, ... (E of them).  grid (ceil(units / 4), ceil(T / TW), B)
template <int E>
__global__ __launch_bounds__(256) void k_delta_inputs(DeltaRows a)
{
    const int lane = threadIdx.x & 63, u = blockIdx.x * 4 + (threadIdx.x >> 6), t0 = blockIdx.y * TW, b = blockIdx.z;
    const int qd = a.KV * a.dim, vd = a.H * a.vdim, m0 = b * a.r.T + t0, nt = min(TW, a.r.T - t0);
    if (u >= a.KV + (vd + 63) / 64) return;
    if (u < a.KV) {
        int ch[2 * E], col[2 * E];
        bool in[2 * E];
        float y[TW][2 * E];
#pragma unroll
        for (int e = 0; e < E; e++) {
            const int d = lane + 64 * e;
            in[e] = in[E + e] = d < a.dim;
            ch[e] = u * a.dim + d; col[e] = a.o_q + ch[e];
            ch[E + e] = qd + u * a.dim + d; col[E + e] = a.o_k + u * a.dim + d;
        }
        conv_tokens<2 * E>(a, b, t0, ch, col, in, y);
        float iq[TW], ik[TW];
#pragma unroll
        for (int i = 0; i < TW; i++) {
            float sq = 0.f, sk = 0.f;
#pragma unroll
            for (int e = 0; e < E; e++) { sq += y[i][e] * y[i][e]; sk += y[i][E + e] * y[i][E + e]; }
            iq[i] = wave_total(sq); ik[i] = wave_total(sk);
        }
#pragma unroll
        for (int i = 0; i < TW; i++) {
            if (i >= nt) break;
            const float fq = 1.f / (sqrtf(iq[i] + 1e-6f) * sqrtf((float)a.dim)), fk = 1.f / sqrtf(ik[i] + 1e-6f);
            const size_t o = ((size_t)(m0 + i) * a.KV + u) * a.dim + lane;
#pragma unroll
            for (int e = 0; e < E; e++)
                if (in[e]) { a.q[o + 64 * e] = y[i][e] * fq; a.k[o + 64 * e] = y[i][E + e] * fk; }
        }
        return;
    }
    const int c = (u - a.KV) * 64 + lane, ch[1] = {2 * qd + c}, col[1] = {a.o_v + c};
    const bool in[1] = {c < vd};
    float y[TW][1];
    conv_tokens<1>(a, b, t0, ch, col, in, y);
#pragma unroll
    for (int i = 0; i < TW; i++) if (i < nt && in[0]) a.v[(size_t)(m0 + i) * vd + c] = y[i][0];
}

// ---------------------------------------------------------------- tokens in groups of four
//
// Four tokens are taken through the recurrence together.  With S the state ahead of them, d(j, i) the decay between
// writing token j and reading token i (the product of the decays of j + 1 .. i) and d(0-, i) the one from S to i:
//     p_i = S^T (d(0-, i) k_i)          w_i = S^T (d(0-, i) q_i)
//     u_i = beta_i (v_i - p_i - sum_{j < i} A_ij u_j)      A_ij = k_i . d(j, i) k_j
//     o_i = w_i + sum_{j <= i} B_ij u_j                    B_ij = q_i . d(j, i) k_j
//     S  <- d(0-, 3) S + sum_j d(j, 3) k_j u_j^T
// which is the token-by-token recurrence with the sums written out: all eight products with the state run side by side,
// and the state is written once.  The numbers that do not depend on the state are made ahead, 32 per group and head:
//     0 .. 3 beta | 4 .. 9 A10 A20 A21 A30 A31 A32 | 12 .. 21 B00 B10 B11 B20 B21 B22 B30 B31 B32 B33
//     | 24 .. 27 d(0-, i) | 28 .. 31 d(i, 3)  (the last two with one decay per head only)
constexpr int GT = 4, GS = 32;

// One wave per (group, head): decays, step sizes and the pair products.  grid (ceil(H / 4), groups, B)
template <int E, int PC>
__global__ __launch_bounds__(256) void k_delta_pairs(DeltaRows a)
{
    const int lane = threadIdx.x & 63, h = blockIdx.x * 4 + (threadIdx.x >> 6), grp = blockIdx.y, b = blockIdx.z, T = a.r.T;
    if (h >= a.H) return;
    const int kvh = h / (a.H / a.KV), t0 = grp * GT, nt = min(GT, T - t0);
    const size_t m0 = (size_t)b * T + t0;
    float k[GT][E], q[GT][E], g[GT][E], gh[GT];
    const float ae = a.a_exp[h];
#pragma unroll
    for (int i = 0; i < GT; i++) {
        gh[i] = 1.f;
        if (!PC && i < nt) gh[i] = expf(-ae * softplus(a.cin[(m0 + i) * a.ldc + a.o_a + h] + a.dt_bias[h]));
#pragma unroll
        for (int e = 0; e < E; e++) {
            const int d = lane + 64 * e;
            const bool in = d < a.dim && i < nt;
            const size_t o = ((m0 + i) * a.KV + kvh) * a.dim + d;
            k[i][e] = in ? a.k[o] : 0.f;
            q[i][e] = in ? a.q[o] : 0.f;
            g[i][e] = gh[i];
            if (PC && in) {
                const size_t og = ((m0 + i) * a.H + h) * a.dim + d;
                g[i][e] = expf(-ae * softplus(a.a2[og] + a.dt_bias[h * a.dim + d]));
                a.g[og] = g[i][e];
            }
        }
    }
    float A[6], B[10];
    int na = 0, nb = 0;
#pragma unroll
    for (int i = 0; i < GT; i++)
#pragma unroll
        for (int j = 0; j <= i; j++) {
            float sa = 0.f, sb = 0.f;
#pragma unroll
            for (int e = 0; e < E; e++) {
                float kj = k[j][e];
#pragma unroll
                for (int x = j + 1; x <= i; x++) kj *= g[x][e];
                sa = fmaf(k[i][e], kj, sa); sb = fmaf(q[i][e], kj, sb);
            }
            if (j < i) A[na++] = wave_total(sa);
            B[nb++] = wave_total(sb);
        }
    // lane n keeps number n
    float mine = 0.f;
#pragma unroll
    for (int i = 0; i < GT; i++) {
        if (lane == i && i < nt) mine = sigmoid(a.cin[(m0 + i) * a.ldc + a.o_b + h]);
        if (!PC) {
            float c = 1.f, r = 1.f;
#pragma unroll
            for (int x = 0; x < GT; x++) { if (x <= i) c *= gh[x]; else r *= gh[x]; }
            if (lane == 24 + i) mine = c;
            if (lane == 28 + i) mine = r;
        }
    }
#pragma unroll
    for (int n = 0; n < 6; n++) if (lane == 4 + n) mine = A[n];
#pragma unroll
    for (int n = 0; n < 10; n++) if (lane == 12 + n) mine = B[n];
    if (lane < GS) a.pairs[(((size_t)b * ((T + GT - 1) / GT) + grp) * a.H + h) * GS + lane] = mine;
}

// The recurrence.  The columns of a head's state (one per value channel) do not meet: a column is G lanes of a wave, each
// with R of its rows -- lane l of the group has rows 4 l .. 4 l + 3 of every block of 4 G -- so no token costs a barrier.
// Tokens are staged through LDS TC at a time with the decays already on the keys and queries, the next two stages on their
// way in registers; a group's LDS reads are issued one group ahead.  The lane numbered like a token keeps its output until the
// stage is over.
// grid (column blocks of 256 / G, H, B), block 256.  VEC: dim is a multiple of 4 (16-byte loads).
template <int G, int R, int PC, int VEC>
__global__ __launch_bounds__(256) void k_delta_scan(DeltaRows a)
{
    constexpr int TC = 16, NG = TC / GT, DP = G * R, COLS = 256 / G, RB = R / 4;
    constexpr int NC = (TC * COLS + 255) / 256, NK = (TC + G - 1) / G;
    static_assert(DP <= 256, "a thread stages four columns of one group");
    __shared__ float ks[2][TC * DP], qs[2][TC * DP], us[2][PC ? TC * DP : 4], gs[2][PC ? NG * DP : 4];
    __shared__ float vs[2][COLS * TC], ps[2][NG * GS];
    const int tid = threadIdx.x, l = tid % G, col = tid / G;
    const int h = blockIdx.y, b = blockIdx.z, kvh = h / (a.H / a.KV), T = a.r.T, groups = (T + GT - 1) / GT;
    const int j0 = blockIdx.x * COLS, j = j0 + col;
    const size_t r0 = (size_t)b * T;
    float S[R];
    float *Sg = a.S + (((size_t)b * a.H + h) * a.vdim + min(j, a.vdim - 1)) * a.dim;
#pragma unroll
    for (int e = 0; e < R; e++) {
        const int d = (e >> 2) * 4 * G + 4 * l + (e & 3);
        S[e] = (a.r.pos > 0 && d < a.dim) ? Sg[d] : 0.f;  // position 0 starts from nothing, whatever the state held
    }
    // staging: a thread brings four columns of the four tokens of one group (threads from DP on repeat others' reads and
    // park nothing).  Two register sets, a stage's loads are asked for two stages ahead.  Every load is unconditional, past
    // the end for the last token again: under a condition the compiler could not tell the two sets' loads apart and would
    // wait for both.  What lies past the end is taken out when it is parked: no key, no step, decay 1.
    const int sd = (tid % (DP / 4)) * 4, sgrp = tid / (DP / 4) % NG;
    struct Stage { float4 k[GT], q[GT], g[PC ? GT : 1]; float v[NC], p; };
    auto at = [](const float *base, uint32_t i) __attribute__((always_inline)) { return reinterpret_cast<const float *>(reinterpret_cast<const char *>(base) + 4u * i); };
    auto load4 = [&](const float *base, uint32_t i) __attribute__((always_inline)) {
        if (VEC) return *reinterpret_cast<const float4 *>(at(base, i));
        const uint32_t last = (uint32_t)(a.dim - 1 - min(sd, a.dim - 1));
        return make_float4(*at(base, i), *at(base, i + min(1u, last)), *at(base, i + min(2u, last)), *at(base, i + min(3u, last)));
    };
    const uint32_t kq0 = (uint32_t)((r0 * a.KV + kvh) * a.dim + min(sd, a.dim - (VEC ? 4 : 1)));
    const uint32_t g0 = (uint32_t)((r0 * a.H + h) * a.dim + min(sd, a.dim - (VEC ? 4 : 1)));
    auto fetch = [&](Stage &x, int t0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < GT; i++) {
            const uint32_t t = (uint32_t)min(t0 + sgrp * GT + i, T - 1);
            const uint32_t o = kq0 + t * (uint32_t)(a.KV * a.dim);
            x.k[i] = load4(a.k, o); x.q[i] = load4(a.q, o);
            if (PC) x.g[PC ? i : 0] = load4(a.g, g0 + t * (uint32_t)(a.H * a.dim));
        }
#pragma unroll
        for (int i = 0; i < NC; i++) {
            const int e = tid + 256 * i, t = e / COLS % TC, c = e % COLS;
            x.v[i] = *at(a.v, (uint32_t)(((r0 + min(t0 + t, T - 1)) * a.H + h) * a.vdim + min(j0 + c, a.vdim - 1)));
        }
        const int grp = min(t0 / GT + tid / GS % NG, groups - 1);
        x.p = *at(a.pairs, (uint32_t)((((size_t)b * groups + grp) * a.H + h) * GS + tid % GS));
    };
    auto mul4 = [](const float4 &x, const float4 &y) __attribute__((always_inline)) { return make_float4(x.x * y.x, x.y * y.y, x.z * y.z, x.w * y.w); };
    auto park = [&](const Stage &x, int t0, int s) __attribute__((always_inline)) {
        if (tid < DP) {
            const float4 one = make_float4(1.f, 1.f, 1.f, 1.f);
            float4 c = one, r = one, k[GT], g[GT];
#pragma unroll
            for (int i = 0; i < GT; i++) {
                const bool in = t0 + sgrp * GT + i < T;
                const float f0 = in && sd < a.dim ? 1.f : 0.f, f1 = in && (VEC ? sd : sd + 1) < a.dim ? 1.f : 0.f;
                const float f2 = in && (VEC ? sd : sd + 2) < a.dim ? 1.f : 0.f, f3 = in && (VEC ? sd : sd + 3) < a.dim ? 1.f : 0.f;
                const float4 f = make_float4(f0, f1, f2, f3);
                k[i] = mul4(x.k[i], f);
                g[i] = PC && in ? x.g[PC ? i : 0] : one;
                c = mul4(c, g[i]);
                const int to = (sgrp * GT + i) * DP + sd;
                *reinterpret_cast<float4 *>(&ks[s][to]) = PC ? mul4(k[i], c) : k[i];
                *reinterpret_cast<float4 *>(&qs[s][to]) = PC ? mul4(mul4(x.q[i], f), c) : mul4(x.q[i], f);
            }
            if (PC) {
                *reinterpret_cast<float4 *>(&gs[s][sgrp * DP + sd]) = c;
#pragma unroll
                for (int i = GT - 1; i >= 0; i--) {
                    *reinterpret_cast<float4 *>(&us[s][(sgrp * GT + i) * DP + sd]) = mul4(k[i], r);
                    r = mul4(r, g[i]);
                }
            }
        }
#pragma unroll
        for (int i = 0; i < NC; i++) { const int e = tid + 256 * i, t = e / COLS, c = e % COLS; if (t < TC) vs[s][c * TC + t] = x.v[i]; }
        if (tid < NG * GS) ps[s][tid] = x.p;              // (step sizes past the end are zero already)
    };
    struct Group { float4 k[GT][RB], q[GT][RB]; };
    auto read = [&](Group &x, int s, int grp) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < GT; i++)
#pragma unroll
            for (int r = 0; r < RB; r++) {
                const int at = (grp * GT + i) * DP + r * 4 * G + 4 * l;
                x.k[i][r] = *reinterpret_cast<const float4 *>(&ks[s][at]);
                x.q[i][r] = *reinterpret_cast<const float4 *>(&qs[s][at]);
            }
    };
    auto dot = [&](const float4 (&x)[RB]) __attribute__((always_inline)) {
        float y[RB];
#pragma unroll
        for (int r = 0; r < RB; r++) y[r] = fmaf(S[4 * r + 3], x[r].w, fmaf(S[4 * r + 2], x[r].z, fmaf(S[4 * r + 1], x[r].y, S[4 * r] * x[r].x)));
#pragma unroll
        for (int r = 1; r < RB; r++) y[0] += y[r];
        return y[0];
    };
    float keep[NK];
    auto take = [&](const Group &x, int s, int grp) __attribute__((always_inline)) {
        const float4 *n = reinterpret_cast<const float4 *>(&ps[s][grp * GS]);
        const float4 be = n[0], a0 = n[1], a1 = n[2], b0 = n[3], b1 = n[4], b2 = n[5];
        const float4 v = *reinterpret_cast<const float4 *>(&vs[s][col * TC + grp * GT]);
        float p[GT], w[GT];
#pragma unroll
        for (int i = 0; i < GT; i++) { p[i] = dot(x.k[i]); w[i] = dot(x.q[i]); }
#pragma unroll
        for (int i = 0; i < GT; i++) { p[i] = group_sum<G>(p[i]); w[i] = group_sum<G>(w[i]); }
        float u[GT];
        float4 dr = make_float4(1.f, 1.f, 1.f, 1.f);
        float all = 1.f;
        if (!PC) {
            const float4 dc = n[6];
            dr = n[7];
            p[0] *= dc.x; p[1] *= dc.y; p[2] *= dc.z; p[3] *= dc.w;
            w[0] *= dc.x; w[1] *= dc.y; w[2] *= dc.z; w[3] *= dc.w;
            all = dc.w;
        }
        u[0] = be.x * (v.x - p[0]);
        u[1] = be.y * (v.y - p[1] - a0.x * u[0]);
        u[2] = be.z * (v.z - p[2] - a0.y * u[0] - a0.z * u[1]);
        u[3] = be.w * (v.w - p[3] - a0.w * u[0] - a1.x * u[1] - a1.y * u[2]);
        const float o[GT] = {fmaf(b0.x, u[0], w[0]), fmaf(b0.z, u[1], fmaf(b0.y, u[0], w[1])),
                             fmaf(b1.y, u[2], fmaf(b1.x, u[1], fmaf(b0.w, u[0], w[2]))),
                             fmaf(b2.y, u[3], fmaf(b2.x, u[2], fmaf(b1.w, u[1], fmaf(b1.z, u[0], w[3]))))};
        if (!PC) { u[0] *= dr.x; u[1] *= dr.y; u[2] *= dr.z; u[3] *= dr.w; }
#pragma unroll
        for (int r = 0; r < RB; r++) {
            float4 g = make_float4(all, all, all, all);
            if (PC) g = *reinterpret_cast<const float4 *>(&gs[s][grp * DP + r * 4 * G + 4 * l]);
            float *z = &S[4 * r];
            z[0] *= g.x; z[1] *= g.y; z[2] *= g.z; z[3] *= g.w;
#pragma unroll
            for (int i = 0; i < GT; i++) {
                const float4 k = PC ? *reinterpret_cast<const float4 *>(&us[s][PC ? (grp * GT + i) * DP + r * 4 * G + 4 * l : 0]) : x.k[i][r];
                z[0] = fmaf(k.x, u[i], z[0]); z[1] = fmaf(k.y, u[i], z[1]); z[2] = fmaf(k.z, u[i], z[2]); z[3] = fmaf(k.w, u[i], z[3]);
            }
        }
#pragma unroll
        for (int i = 0; i < GT; i++) {
            const int t = grp * GT + i;
            keep[t / G] = l == t % G ? o[i] : keep[t / G];
        }
    };
    Stage even, odd;
    auto stage = [&](int t0, int s, Stage &ahead, const Stage &next) __attribute__((always_inline)) {
        fetch(ahead, t0 + 2 * TC);
#pragma unroll
        for (int i = 0; i < NK; i++) keep[i] = 0.f;
        Group x[2];
        read(x[0], s, 0);
#pragma unroll
        for (int grp = 0; grp < NG; grp++) {
            if (t0 + grp * GT >= T) break;                // uniform
            if (grp + 1 < NG) read(x[(grp + 1) & 1], s, grp + 1);
            take(x[grp & 1], s, grp);
        }
        park(next, t0 + TC, s ^ 1);                       // the other stage: its readers passed the barrier before this one
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int t = i * G + l;
            if (t < TC && t0 + t < T && j < a.vdim) a.o[((r0 + t0 + t) * a.H + h) * a.vdim + j] = keep[i];
        }
        __syncthreads();
    };
    fetch(even, 0);
    fetch(odd, TC);
    park(even, 0, 0);
    __syncthreads();
    for (int t0 = 0; t0 < T; t0 += 2 * TC) {
        stage(t0, 0, even, odd);
        if (t0 + TC < T) stage(t0 + TC, 1, odd, even);
    }
    if (j < a.vdim)
#pragma unroll
        for (int e = 0; e < R; e++) {
            const int d = (e >> 2) * 4 * G + 4 * l + (e & 3);
            if (d < a.dim) Sg[d] = S[e];
        }
}

// The last `taps` inputs of this step's convolutions into the state's ring.  grid (ceil(channels / 256), taps, B)
__global__ __launch_bounds__(256) void k_conv_keep(DeltaRows a)
{
    const int ch = blockIdx.x * 256 + threadIdx.x, i = blockIdx.y, b = blockIdx.z, T = a.r.T;
    const int qd = a.KV * a.dim, C = 2 * qd + a.H * a.vdim, t = T - 1 - i;
    if (ch >= C || t < 0) return;
    const int col = ch < qd ? a.o_q + ch : ch < 2 * qd ? a.o_k + ch - qd : a.o_v + ch - 2 * qd;
    a.conv[((size_t)b * a.taps + (a.r.pos + t) % a.taps) * C + ch] = a.cin[(size_t)(b * T + t) * a.ldc + col];
}

// One workgroup per row: mixer output with its head norm and gate | squared ReLU of the shared expert's up product.
__global__ __launch_bounds__(256) void k_cat_rows(CatRows a)
{
    extern __shared__ float row[];                        // [ldk]
    __shared__ float sm[16];
    const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    for (int i = a.H * a.vdim + tid; i < a.ldk; i += 256) row[i] = 0.f;
    if (a.g_out) {
        for (int h = wave; h < a.H; h += 4) {
            const float *o = a.o + ((size_t)m * a.H + h) * a.vdim, *gt = a.gate + (size_t)m * a.ld_gate + h * a.vdim;
            float ss = 0.f;
            for (int d = lane; d < a.vdim; d += 64) ss += o[d] * o[d];
            const float inv = 1.f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
            for (int d = lane; d < a.vdim; d += 64) row[h * a.vdim + d] = o[d] * inv * a.g_out[d] * (a.gate_silu ? silu(gt[d]) : sigmoid(gt[d]));
        }
    } else
        for (int i = tid; i < a.H * a.vdim; i += 256) row[i] = a.o[(size_t)m * a.H * a.vdim + i];
    __syncthreads();                                      // the zeros are down before the shared part overwrites some
    for (int i = tid; i < a.shared_ff; i += 256) row[a.o_sh + i] = relu2(a.shared[(size_t)m * a.ld_shared + i]);
    __syncthreads();
    if (a.cat)
        for (int i = tid; i < a.ldk; i += 256) a.cat[(size_t)m * a.ldk + i] = row[i];
    if (a.a16) {
        float mx = 0.f;
        for (int i = tid; i < a.ldk; i += 256) mx = fmaxf(mx, fabsf(row[i]));
        const float s = row_scale_for(block_max(mx, sm));
        store_row_f16(row, a.ldk, a.a16, m, tiled_kb(a.ldk), s);
        if (tid == 0) a.inv[m] = 1.f / s;
    }
}

}  // namespace

int delta_groups(int T) { return (T + GT - 1) / GT; }
size_t delta_pair_floats(int B, int T, int H) { return (size_t)B * delta_groups(T) * H * GS; }

void launch_delta_inputs(const DeltaRows &a)
{
    const dim3 grid((a.KV + (a.H * a.vdim + 63) / 64 + 3) / 4, (a.r.T + TW - 1) / TW, a.r.B), pgrid((a.H + 3) / 4, delta_groups(a.r.T), a.r.B);
#define INPUTS(E_) do { \
    LAUNCH(k_delta_inputs<E_>, grid, dim3(256), 0, a); \
    if (a.per_channel) LAUNCH((k_delta_pairs<E_, 1>), pgrid, dim3(256), 0, a); else LAUNCH((k_delta_pairs<E_, 0>), pgrid, dim3(256), 0, a); } while (0)
    if (a.dim <= 64) INPUTS(1); else if (a.dim <= 128) INPUTS(2); else INPUTS(4);
#undef INPUTS
}

void launch_delta_scan(const DeltaRows &a)
{
    // eight rows per lane; four where the columns would otherwise leave most of the SIMDs without a wave
    const int g8 = a.dim <= 32 ? 4 : a.dim <= 64 ? 8 : a.dim <= 128 ? 16 : 32;
    const bool few = (long)a.r.B * a.H * a.vdim * g8 / 64 <= 2 * num_cus() && a.dim <= 128;
    const int G = few ? 2 * g8 : g8, cols = 256 / G;
    const dim3 grid((a.vdim + cols - 1) / cols, a.H, a.r.B);
#define SCAN(G_, R_) do { \
    if (a.dim % 4 == 0) { if (a.per_channel) LAUNCH((k_delta_scan<G_, R_, 1, 1>), grid, dim3(256), 0, a); else LAUNCH((k_delta_scan<G_, R_, 0, 1>), grid, dim3(256), 0, a); } \
    else { if (a.per_channel) LAUNCH((k_delta_scan<G_, R_, 1, 0>), grid, dim3(256), 0, a); else LAUNCH((k_delta_scan<G_, R_, 0, 0>), grid, dim3(256), 0, a); } } while (0)
    if (few) { if (G == 8) SCAN(8, 4); else if (G == 16) SCAN(16, 4); else SCAN(32, 4); }
    else if (G == 4) SCAN(4, 8); else if (G == 8) SCAN(8, 8); else if (G == 16) SCAN(16, 8); else SCAN(32, 8);
#undef SCAN
    const int C = 2 * a.KV * a.dim + a.H * a.vdim;
    LAUNCH(k_conv_keep, dim3((C + 255) / 256, a.taps, a.r.B), dim3(256), 0, a);
}

void launch_cat_rows(const CatRows &a, int rows) { LAUNCH(k_cat_rows, dim3(rows), dim3(256), (size_t)a.ldk * 4, a); }

}  // namespace lmhip
