// Gated delta rule: short causal convolutions, unit norms, decays, the recurrence over tokens, the gated head norm.
// Everything here is fp32.
#include "stack.h"
#include "delta_rows.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

// silu of the convolution at one channel for the tokens t0 .. t0 + TW - 1 of sequence b, one after the other: `use(i, value)`.
// Up to four taps the inputs slide through registers, each read once; more taps are gathered token by token.
constexpr int TW = 8;        // tokens per wave
template <int NE, typename F>
__device__ __forceinline__ void conv_tokens(const DeltaRows &a, int b, int t0, const int (&ch)[NE], const int (&col)[NE], const bool (&in)[NE], F use)
{
    const int T = a.r.T, nt = min(TW, T - t0), C = 2 * a.KV * a.dim + a.H * a.vdim;
    if (a.taps <= 4) {
        float f[NE][4], x[NE][TW + 3];
#pragma unroll
        for (int e = 0; e < NE; e++)
#pragma unroll
            for (int i = 0; i < 4; i++) f[e][i] = in[e] && i >= 4 - a.taps ? a.filters[(size_t)ch[e] * a.taps + i - (4 - a.taps)] : 0.f;
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
        for (int i = 0; i < TW; i++) {
            if (i >= nt) break;
            float y[NE];
#pragma unroll
            for (int e = 0; e < NE; e++) y[e] = in[e] ? silu(fmaf(f[e][3], x[e][i + 3], fmaf(f[e][2], x[e][i + 2], fmaf(f[e][1], x[e][i + 1], f[e][0] * x[e][i])))) : 0.f;
            use(i, y);
        }
    } else
        for (int i = 0; i < nt; i++) {
            float y[NE];
#pragma unroll
            for (int e = 0; e < NE; e++) y[e] = in[e] ? silu(conv_at(a, b * T + t0 + i, ch[e], col[e])) : 0.f;
            use(i, y);
        }
}

// One wave per (unit, TW tokens): units 0 .. KV-1 finish q and k of a key head (and their dot product), the next H the value
// head, its step size and its decay.  A lane holds channels lane, lane + 64, ... (E of them).  grid (ceil(units / 4),
// ceil(T / TW), B)
template <int E>
__global__ __launch_bounds__(256) void k_delta_inputs(DeltaRows a)
{
    const int lane = threadIdx.x & 63, u = blockIdx.x * 4 + (threadIdx.x >> 6), t0 = blockIdx.y * TW, b = blockIdx.z;
    if (u >= a.KV + a.H) return;
    const int qd = a.KV * a.dim, m0 = b * a.r.T + t0;
    if (u < a.KV) {
        int ch[2 * E], col[2 * E];
        bool in[2 * E];
#pragma unroll
        for (int e = 0; e < E; e++) {
            const int d = lane + 64 * e;
            in[e] = in[E + e] = d < a.dim;
            ch[e] = u * a.dim + d; col[e] = a.o_q + ch[e];
            ch[E + e] = qd + u * a.dim + d; col[E + e] = a.o_k + u * a.dim + d;
        }
        conv_tokens<2 * E>(a, b, t0, ch, col, in, [&](int i, const float (&y)[2 * E]) {
            float sq = 0.f, sk = 0.f, dot = 0.f;
#pragma unroll
            for (int e = 0; e < E; e++) { sq += y[e] * y[e]; sk += y[E + e] * y[E + e]; dot += y[e] * y[E + e]; }
            sq = wave_total(sq); sk = wave_total(sk); dot = wave_total(dot);
            const float iq = 1.f / (sqrtf(sq + 1e-6f) * sqrtf((float)a.dim)), ik = 1.f / sqrtf(sk + 1e-6f);
            const size_t o = ((size_t)(m0 + i) * a.KV + u) * a.dim;
#pragma unroll
            for (int e = 0; e < E; e++)
                if (in[e]) { a.q[o + lane + 64 * e] = y[e] * iq; a.k[o + lane + 64 * e] = y[E + e] * ik; }
            if (lane == 0) a.kq[(size_t)(m0 + i) * a.KV + u] = dot * iq * ik;
        });
        return;
    }
    const int h = u - a.KV;
    for (int d0 = 0; d0 < a.vdim; d0 += 64) {
        const int d = d0 + lane, ch[1] = {2 * qd + h * a.vdim + d}, col[1] = {a.o_v + h * a.vdim + d};
        const bool in[1] = {d < a.vdim};
        conv_tokens<1>(a, b, t0, ch, col, in, [&](int i, const float (&y)[1]) { if (in[0]) a.v[((size_t)(m0 + i) * a.H + h) * a.vdim + d] = y[0]; });
    }
    const int nt = min(TW, a.r.T - t0);
    if (lane < nt) {
        const float *row = a.cin + (size_t)(m0 + lane) * a.ldc;
        a.beta[(size_t)(m0 + lane) * a.H + h] = sigmoid(row[a.o_b + h]);
        if (!a.per_channel) a.g[(size_t)(m0 + lane) * a.H + h] = expf(-a.a_exp[h] * softplus(row[a.o_a + h] + a.dt_bias[h]));
    }
    if (a.per_channel)
        for (int d = lane; d < a.dim; d += 64) {
            const float ae = a.a_exp[h], bias = a.dt_bias[h * a.dim + d];
#pragma unroll
            for (int i = 0; i < TW; i++) {
                if (i >= nt) break;
                const size_t o = ((size_t)(m0 + i) * a.H + h) * a.dim + d;
                a.g[o] = expf(-ae * softplus(a.a2[o] + bias));
            }
        }
}

// The recurrence.  The columns of a head's state (one per value channel) do not meet: a column is G lanes of a wave, each
// with R of its rows -- lane l of the group has rows 4 l .. 4 l + 3 of every block of 4 G -- so a token costs no barrier:
// with both dot products taken before the update (o = (g S)^T q + u (k . q), the read-out after the write) they are reduced
// side by side.  Tokens are staged through LDS TC at a time, the next TC on their way in registers; a token's LDS reads are
// issued two tokens ahead.  The lane numbered like the token keeps its output until the stage is over.
// grid (column blocks of 256 / G, H, B), block 256.  VEC: dim is a multiple of 4 (16-byte loads).
template <int G, int R, int PC, int VEC>
__global__ __launch_bounds__(256) void k_delta_scan(DeltaRows a)
{
    constexpr int TC = 16, DP = G * R, COLS = 256 / G, RB = R / 4;
    constexpr int NV = (TC * DP / 4 + 255) / 256;         // 16-byte pieces per thread and array of one stage
    constexpr int NC = (TC * COLS + 255) / 256, NK = (TC + G - 1) / G;
    __shared__ float ks[2][TC * DP], qs[2][TC * DP], gs[2][PC ? TC * DP : TC];
    __shared__ float vs[2][TC * COLS];
    __shared__ float2 bs[2][TC];                          // (step size, k . q)
    const int tid = threadIdx.x, l = tid % G, col = tid / G;
    const int h = blockIdx.y, b = blockIdx.z, kvh = h / (a.H / a.KV), T = a.r.T;
    const int j0 = blockIdx.x * COLS, j = j0 + col;
    const size_t r0 = (size_t)b * T;
    float S[R];
    float *Sg = a.S + (((size_t)b * a.H + h) * a.vdim + min(j, a.vdim - 1)) * a.dim;
#pragma unroll
    for (int e = 0; e < R; e++) {
        const int d = (e >> 2) * 4 * G + 4 * l + (e & 3);
        S[e] = (a.r.pos > 0 && d < a.dim) ? Sg[d] : 0.f;  // position 0 starts from nothing, whatever the state held
    }
    float4 kr[NV], qr[NV], gr[PC ? NV : 1];
    float vr[NC], gsr = 0.f;
    float2 br = make_float2(0.f, 0.f);
    // tokens past the end leave the state alone: no key, no step, decay 1
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int e = (tid + 256 * i) * 4, t = e / DP, d = e % DP;
            const bool in = t0 + t < T && t < TC && d < a.dim;
            kr[i] = qr[i] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (PC) gr[PC ? i : 0] = make_float4(1.f, 1.f, 1.f, 1.f);
            if (in) {
                const float *k = a.k + ((r0 + t0 + t) * a.KV + kvh) * a.dim + d, *q = a.q + ((r0 + t0 + t) * a.KV + kvh) * a.dim + d;
                const float *g = PC ? a.g + ((r0 + t0 + t) * a.H + h) * a.dim + d : nullptr;
                if (VEC) {
                    kr[i] = *reinterpret_cast<const float4 *>(k); qr[i] = *reinterpret_cast<const float4 *>(q);
                    if (PC) gr[PC ? i : 0] = *reinterpret_cast<const float4 *>(g);
                } else {
                    float *kd = &kr[i].x, *qd = &qr[i].x, *gd = &gr[PC ? i : 0].x;
#pragma unroll
                    for (int u = 0; u < 4; u++) if (d + u < a.dim) { kd[u] = k[u]; qd[u] = q[u]; if (PC) gd[u] = g[u]; }
                }
            }
        }
#pragma unroll
        for (int i = 0; i < NC; i++) {
            const int e = tid + 256 * i, t = e / COLS, c = e % COLS;
            vr[i] = (t < TC && t0 + t < T && j0 + c < a.vdim) ? a.v[((r0 + t0 + t) * a.H + h) * a.vdim + j0 + c] : 0.f;
        }
        if (tid < TC) {
            br = make_float2(0.f, 0.f); gsr = 1.f;
            if (t0 + tid < T) {
                const size_t m = r0 + t0 + tid;
                br = make_float2(a.beta[m * a.H + h], a.kq[m * a.KV + kvh]);
                if (!PC) gsr = a.g[m * a.H + h];
            }
        }
    };
    auto park = [&](int s) {
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int e = (tid + 256 * i) * 4;
            if (e < TC * DP) {
                *reinterpret_cast<float4 *>(&ks[s][e]) = kr[i]; *reinterpret_cast<float4 *>(&qs[s][e]) = qr[i];
                if (PC) *reinterpret_cast<float4 *>(&gs[s][e]) = gr[PC ? i : 0];
            }
        }
#pragma unroll
        for (int i = 0; i < NC; i++) { const int e = tid + 256 * i; if (e < TC * COLS) vs[s][e] = vr[i]; }
        if (tid < TC) { bs[s][tid] = br; if (!PC) gs[s][tid] = gsr; }
    };
    struct Tok { float4 k[RB], q[RB], g[PC ? RB : 1]; float gv, v; float2 b; };
    auto read = [&](Tok &x, int s, int t) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < RB; i++) {
            x.k[i] = *reinterpret_cast<const float4 *>(&ks[s][t * DP + i * 4 * G + 4 * l]);
            x.q[i] = *reinterpret_cast<const float4 *>(&qs[s][t * DP + i * 4 * G + 4 * l]);
            if (PC) x.g[PC ? i : 0] = *reinterpret_cast<const float4 *>(&gs[s][t * DP + i * 4 * G + 4 * l]);
        }
        if (!PC) x.gv = gs[s][t];
        x.v = vs[s][t * COLS + col];
        x.b = bs[s][t];
    };
    auto token = [&](const Tok &x) __attribute__((always_inline)) -> float {
        float p[RB], w[RB];
#pragma unroll
        for (int i = 0; i < RB; i++) {
            const float k[4] = {x.k[i].x, x.k[i].y, x.k[i].z, x.k[i].w}, q[4] = {x.q[i].x, x.q[i].y, x.q[i].z, x.q[i].w};
            const float g[4] = {PC ? x.g[PC ? i : 0].x : x.gv, PC ? x.g[PC ? i : 0].y : x.gv, PC ? x.g[PC ? i : 0].z : x.gv, PC ? x.g[PC ? i : 0].w : x.gv};
#pragma unroll
            for (int e = 0; e < 4; e++) S[4 * i + e] *= g[e];
            p[i] = S[4 * i] * k[0]; w[i] = S[4 * i] * q[0];
#pragma unroll
            for (int e = 1; e < 4; e++) { p[i] = fmaf(S[4 * i + e], k[e], p[i]); w[i] = fmaf(S[4 * i + e], q[e], w[i]); }
        }
#pragma unroll
        for (int i = 1; i < RB; i++) { p[0] += p[i]; w[0] += w[i]; }
        const float ps = group_sum<G>(p[0]), ws = group_sum<G>(w[0]);
        const float u = x.b.x * (x.v - ps);
#pragma unroll
        for (int i = 0; i < RB; i++) {
            const float k[4] = {x.k[i].x, x.k[i].y, x.k[i].z, x.k[i].w};
#pragma unroll
            for (int e = 0; e < 4; e++) S[4 * i + e] = fmaf(k[e], u, S[4 * i + e]);
        }
        return fmaf(u, x.b.y, ws);
    };
    fetch(0);
    park(0);
    __syncthreads();
    for (int t0 = 0, s = 0; t0 < T; t0 += TC, s ^= 1) {
        if (t0 + TC < T) fetch(t0 + TC);
        float keep[NK];
#pragma unroll
        for (int i = 0; i < NK; i++) keep[i] = 0.f;
        if (T - t0 >= TC) {
            Tok x[3];
            read(x[0], s, 0); read(x[1], s, 1);
#pragma unroll
            for (int t = 0; t < TC; t++) {
                if (t + 2 < TC) read(x[(t + 2) % 3], s, t + 2);
                const float o = token(x[t % 3]);
                keep[t / G] = l == t % G ? o : keep[t / G];
            }
        } else {
#pragma unroll 1
            for (int t = 0; t < T - t0; t++) {
                Tok x;
                read(x, s, t);
                const float o = token(x);
#pragma unroll
                for (int i = 0; i < NK; i++) if (t == i * G + l) keep[i] = o;
            }
        }
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int t = t0 + i * G + l;
            if (i * G + l < TC && t < T && j < a.vdim) a.o[((r0 + t) * a.H + h) * a.vdim + j] = keep[i];
        }
        if (t0 + TC < T) park(s ^ 1);                     // the other stage: its readers passed the barrier below
        __syncthreads();
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

void launch_delta_inputs(const DeltaRows &a)
{
    const dim3 grid((a.KV + a.H + 3) / 4, (a.r.T + TW - 1) / TW, a.r.B);
    if (a.dim <= 64) LAUNCH(k_delta_inputs<1>, grid, dim3(256), 0, a);
    else if (a.dim <= 128) LAUNCH(k_delta_inputs<2>, grid, dim3(256), 0, a);
    else LAUNCH(k_delta_inputs<4>, grid, dim3(256), 0, a);
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
