// Gated delta rule: short causal convolutions, unit norms, decays, the recurrence over tokens, the gated head norm.
// Everything here is fp32.
#include "stack.h"
#include "rows.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

// Channel ch (q | k | v order) of the convolution at row m: the inputs of this step from the product, older ones from
// the state's ring (the input of position p lies at p % taps), zeros before position 0.
__device__ __forceinline__ float conv_at(const DeltaRows &a, int m, int ch, int in_col)
{
    const int b = m / a.r.T, t = m % a.r.T, C = 2 * a.KV * a.dim + a.H * a.vdim;
    const float *f = a.filters + (size_t)ch * a.taps;
    float s = 0.f;
    for (int i = 0; i < a.taps; i++) {
        const int tt = t - (a.taps - 1) + i, p = a.r.pos + tt;
        if (p < 0) continue;
        const float x = tt >= 0 ? a.cin[(size_t)(b * a.r.T + tt) * a.ldc + in_col] : a.conv[((size_t)b * a.taps + p % a.taps) * C + ch];
        s = fmaf(x, f[i], s);
    }
    return s;
}

// One wave per (row, unit): units 0 .. KV-1 finish q and k of a key head (and their dot product), the next H the value
// head, its step size and its decay.  grid (ceil(units / 4), rows)
__global__ __launch_bounds__(256) void k_delta_inputs(DeltaRows a)
{
    const int lane = threadIdx.x & 63, u = blockIdx.x * 4 + (threadIdx.x >> 6), m = blockIdx.y;
    if (u >= a.KV + a.H) return;
    const int qd = a.KV * a.dim;
    if (u < a.KV) {
        float qv[4], kv[4], sq = 0.f, sk = 0.f, dot = 0.f;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int d = lane + 64 * e;
            qv[e] = kv[e] = 0.f;
            if (d < a.dim) {
                const int ch = u * a.dim + d;
                qv[e] = silu(conv_at(a, m, ch, a.o_q + ch));
                kv[e] = silu(conv_at(a, m, qd + ch, a.o_k + ch));
            }
            sq += qv[e] * qv[e]; sk += kv[e] * kv[e]; dot += qv[e] * kv[e];
        }
        sq = wave_sum(sq); sk = wave_sum(sk); dot = wave_sum(dot);
        const float iq = 1.f / (sqrtf(sq + 1e-6f) * sqrtf((float)a.dim)), ik = 1.f / sqrtf(sk + 1e-6f);
        const size_t o = ((size_t)m * a.KV + u) * a.dim;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int d = lane + 64 * e;
            if (d < a.dim) { a.q[o + d] = qv[e] * iq; a.k[o + d] = kv[e] * ik; }
        }
        if (lane == 0) a.kq[(size_t)m * a.KV + u] = dot * iq * ik;
        return;
    }
    const int h = u - a.KV;
    for (int d = lane; d < a.vdim; d += 64) {
        const int ch = h * a.vdim + d;
        a.v[((size_t)m * a.H + h) * a.vdim + d] = silu(conv_at(a, m, 2 * qd + ch, a.o_v + ch));
    }
    const float *row = a.cin + (size_t)m * a.ldc;
    if (lane == 0) a.beta[(size_t)m * a.H + h] = sigmoid(row[a.o_b + h]);
    if (a.per_channel) {
        for (int d = lane; d < a.dim; d += 64) {
            const size_t i = ((size_t)m * a.H + h) * a.dim + d;
            a.g[i] = expf(-a.a_exp[h] * softplus(a.a2[i] + a.dt_bias[h * a.dim + d]));
        }
    } else if (lane == 0) a.g[(size_t)m * a.H + h] = expf(-a.a_exp[h] * softplus(row[a.o_a + h] + a.dt_bias[h]));
}

// The recurrence.  The columns of a head's state (one per value channel) do not meet: a column is G lanes of a wave,
// each with eight of its rows -- rows 4 l .. 4 l + 3 and those 4 G further, for lane l of the group -- so a token costs
// no barrier: with both dot products taken before the update (o = (g S)^T q + u (k . q), the read-out after the write)
// they are reduced side by side.  Tokens are staged through LDS TC at a time, the next TC on their way in registers.
// grid (column blocks of 256 / G, H, B), block 256.
template <int G, int PC>
__global__ __launch_bounds__(256) void k_delta_scan(DeltaRows a)
{
    constexpr int TC = 16, DP = G * 8, COLS = 256 / G;
    constexpr int NV = TC * DP / 256;                     // floats per thread and array of one stage
    __shared__ float ks[2][TC * DP], qs[2][TC * DP], gs[2][PC ? TC * DP : TC];
    __shared__ float vs[2][TC * COLS], bs[2][TC], kqs[2][TC], os[TC * COLS];
    const int tid = threadIdx.x, l = tid % G, col = tid / G;
    const int h = blockIdx.y, b = blockIdx.z, kvh = h / (a.H / a.KV), T = a.r.T;
    const int j0 = blockIdx.x * COLS, j = j0 + col;
    const size_t r0 = (size_t)b * T;
    float S[8];
    float *Sg = a.S + (((size_t)b * a.H + h) * a.vdim + min(j, a.vdim - 1)) * a.dim;
#pragma unroll
    for (int e = 0; e < 8; e++) {
        const int d = (e >> 2) * 4 * G + 4 * l + (e & 3);
        S[e] = (a.r.pos > 0 && d < a.dim) ? Sg[d] : 0.f;  // position 0 starts from nothing, whatever the state held
    }
    float kr[NV], qr[NV], gr[PC ? NV : 1], vr[(TC * COLS + 255) / 256], br = 0.f, kqr = 0.f, gsr = 0.f;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int e = tid + 256 * i, t = e / DP, d = e % DP, tt = min(t0 + t, T - 1);
            const bool in = d < a.dim;
            const size_t qk = ((r0 + tt) * a.KV + kvh) * a.dim + (in ? d : 0);
            kr[i] = in ? a.k[qk] : 0.f;
            qr[i] = in ? a.q[qk] : 0.f;
            if (PC) gr[PC ? i : 0] = in ? a.g[((r0 + tt) * a.H + h) * a.dim + d] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < (TC * COLS + 255) / 256; i++) {
            const int e = tid + 256 * i, t = e / COLS, c = e % COLS;
            vr[i] = (t < TC && j0 + c < a.vdim) ? a.v[((r0 + min(t0 + t, T - 1)) * a.H + h) * a.vdim + j0 + c] : 0.f;
        }
        if (tid < TC) {
            const size_t m = r0 + min(t0 + tid, T - 1);
            br = a.beta[m * a.H + h];
            kqr = a.kq[m * a.KV + kvh];
            if (!PC) gsr = a.g[m * a.H + h];
        }
    };
    auto park = [&](int s) {
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int e = tid + 256 * i;
            ks[s][e] = kr[i]; qs[s][e] = qr[i];
            if (PC) gs[s][e] = gr[PC ? i : 0];
        }
#pragma unroll
        for (int i = 0; i < (TC * COLS + 255) / 256; i++) { const int e = tid + 256 * i; if (e < TC * COLS) vs[s][e] = vr[i]; }
        if (tid < TC) { bs[s][tid] = br; kqs[s][tid] = kqr; if (!PC) gs[s][tid] = gsr; }
    };
    fetch(0);
    park(0);
    __syncthreads();
    for (int t0 = 0, s = 0; t0 < T; t0 += TC, s ^= 1) {
        if (t0 + TC < T) fetch(t0 + TC);
        const int nt = min(TC, T - t0);
        for (int t = 0; t < nt; t++) {
            const float4 k0 = *reinterpret_cast<const float4 *>(&ks[s][t * DP + 4 * l]), k1 = *reinterpret_cast<const float4 *>(&ks[s][t * DP + 4 * G + 4 * l]);
            const float4 q0 = *reinterpret_cast<const float4 *>(&qs[s][t * DP + 4 * l]), q1 = *reinterpret_cast<const float4 *>(&qs[s][t * DP + 4 * G + 4 * l]);
            const float kk[8] = {k0.x, k0.y, k0.z, k0.w, k1.x, k1.y, k1.z, k1.w};
            const float qq[8] = {q0.x, q0.y, q0.z, q0.w, q1.x, q1.y, q1.z, q1.w};
            if (PC) {
                const float4 g0 = *reinterpret_cast<const float4 *>(&gs[s][t * DP + 4 * l]), g1 = *reinterpret_cast<const float4 *>(&gs[s][t * DP + 4 * G + 4 * l]);
                S[0] *= g0.x; S[1] *= g0.y; S[2] *= g0.z; S[3] *= g0.w; S[4] *= g1.x; S[5] *= g1.y; S[6] *= g1.z; S[7] *= g1.w;
            } else {
                const float g = gs[s][t];
#pragma unroll
                for (int e = 0; e < 8; e++) S[e] *= g;
            }
            float p0 = 0.f, p1 = 0.f, w0 = 0.f, w1 = 0.f;
#pragma unroll
            for (int e = 0; e < 4; e++) {
                p0 = fmaf(S[e], kk[e], p0); p1 = fmaf(S[4 + e], kk[4 + e], p1);
                w0 = fmaf(S[e], qq[e], w0); w1 = fmaf(S[4 + e], qq[4 + e], w1);
            }
            const float p = group_sum<G>(p0 + p1), w = group_sum<G>(w0 + w1);
            const float u = bs[s][t] * (vs[s][t * COLS + col] - p);
#pragma unroll
            for (int e = 0; e < 8; e++) S[e] = fmaf(kk[e], u, S[e]);
            if (l == 0) os[t * COLS + col] = fmaf(u, kqs[s][t], w);
        }
        __syncthreads();                                  // os is whole; stage s has been read by all
        for (int i = tid; i < nt * COLS; i += 256) {
            const int t = i / COLS, c = i % COLS;
            if (j0 + c < a.vdim) a.o[((r0 + t0 + t) * a.H + h) * a.vdim + j0 + c] = os[i];
        }
        if (t0 + TC < T) park(s ^ 1);
        __syncthreads();
    }
    if (j < a.vdim)
#pragma unroll
        for (int e = 0; e < 8; e++) {
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

void launch_delta_inputs(const DeltaRows &a) { LAUNCH(k_delta_inputs, dim3((a.KV + a.H + 3) / 4, a.r.n()), dim3(256), 0, a); }

void launch_delta_scan(const DeltaRows &a)
{
    const int G = a.dim <= 32 ? 4 : a.dim <= 64 ? 8 : a.dim <= 128 ? 16 : 32, cols = 256 / G;
    const dim3 grid((a.vdim + cols - 1) / cols, a.H, a.r.B);
#define SCAN(G_) do { if (a.per_channel) LAUNCH((k_delta_scan<G_, 1>), grid, dim3(256), 0, a); else LAUNCH((k_delta_scan<G_, 0>), grid, dim3(256), 0, a); } while (0)
    if (G == 4) SCAN(4); else if (G == 8) SCAN(8); else if (G == 16) SCAN(16); else SCAN(32);
#undef SCAN
    const int C = 2 * a.KV * a.dim + a.H * a.vdim;
    LAUNCH(k_conv_keep, dim3((C + 255) / 256, a.taps, a.r.B), dim3(256), 0, a);
}

void launch_cat_rows(const CatRows &a, int rows) { LAUNCH(k_cat_rows, dim3(rows), dim3(256), (size_t)a.ldk * 4, a); }

}  // namespace lmhip
