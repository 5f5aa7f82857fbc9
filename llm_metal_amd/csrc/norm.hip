// The row kernels of a layer-by-layer model around its products: embedding rows, the residual sum with the norm that feeds
// a product, the dense feed-forward's activation, rotation tables.
#include "stack.h"
#include "rows.h"
#include "planes.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

__global__ __launch_bounds__(256) void k_embed_rows(const float *__restrict__ emb, const int *__restrict__ tok, float scale,
                                                    float *__restrict__ x, int D, int Dp)
{
    const int m = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
    if (i < Dp) x[(size_t)m * Dp + i] = i < D ? emb[(size_t)tok[m] * D + i] * scale : 0.f;
}

// the same for tokens that travel with the launch
struct FewTokens { int id[STACK_FEW]; };
__global__ __launch_bounds__(256) void k_embed_few(const float *__restrict__ emb, FewTokens tok, float scale, float *__restrict__ x, int D, int Dp)
{
    const int m = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
    if (i < Dp) x[(size_t)m * Dp + i] = i < D ? emb[(size_t)tok.id[m] * D + i] * scale : 0.f;
}

// One workgroup per row; the row waits in LDS between the passes (mean, squared deviations, output).
__global__ __launch_bounds__(256) void k_norm_rows(NormRows a)
{
    extern __shared__ float row[];                        // [Dp]
    __shared__ float sm[32];
    const int m = blockIdx.x, src = a.want ? a.want[m] : m * a.step + a.first, tid = threadIdx.x;
    const size_t off = (size_t)src * a.Dp;
    float sum = 0.f;
    for (int i = tid * 4; i < a.Dp; i += 1024) {
        float4 v = *reinterpret_cast<const float4 *>(a.x + off + i);
        auto add = [&](const float *p, float f) {
            const float4 w = *reinterpret_cast<const float4 *>(p + i);
            v.x = fmaf(w.x, f, v.x); v.y = fmaf(w.y, f, v.y); v.z = fmaf(w.z, f, v.z); v.w = fmaf(w.w, f, v.w);
        };
        if (a.cout) {
            // the two sublayers' sum is formed before it meets the residual
            const float4 r = v;
            v = make_float4(0.f, 0.f, 0.f, 0.f);
            add(a.cout + off, 1.f);
            if (a.ymoe) add(a.ymoe + off, 1.f);
            else if (a.moe_y)
                for (int s = 0; s < a.top; s++) add(a.moe_y + (size_t)a.moe_pos[(size_t)src * a.top + s] * a.Dp, a.route_w[(size_t)src * a.top + s]);
            v.x += r.x; v.y += r.y; v.z += r.z; v.w += r.w;
            if (a.keep) *reinterpret_cast<float4 *>(a.x + off + i) = v;
        }
        *reinterpret_cast<float4 *>(row + i) = v;
        sum += (v.x + v.y) + (v.z + v.w);                 // the padding beyond D holds zeros
    }
    const float mean = block_sum(sum, sm) / (float)a.D;
    float ss = 0.f, mx = 0.f;
    for (int i = tid * 4; i < a.Dp; i += 1024)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const float d = i + e < a.D ? row[i + e] - mean : 0.f;
            ss += d * d;
            const float w = d * a.g[i + e];
            row[i + e] = w;
            mx = fmaxf(mx, fabsf(w));
        }
    block_sum_max(ss, mx, sm);                            // its barriers also publish the row
    const float inv = 1.f / sqrtf(ss / (float)a.D + a.eps);
    if (a.h)
        for (int i = tid; i < a.Dp; i += 256) a.h[(size_t)m * a.Dp + i] = row[i] * inv;
    if (a.a16) {
        const float s = row_scale_for(mx * inv);
        store_row_f16(row, a.Dp, a.a16, m, tiled_kb(a.Dp), s * inv);
        if (tid == 0) a.inv[m] = 1.f / s;
    }
}

// One workgroup per row: the norm behind a sublayer, the residual sum, the norm ahead of the next one.
__global__ __launch_bounds__(256) void k_norms_around(AroundRows a)
{
    extern __shared__ float row[];                        // [Dp]
    __shared__ float sm[32];
    const int m = xcd_block_row(blockIdx.x, gridDim.x), src = a.want ? a.want[m] : m * a.step + a.first, tid = threadIdx.x;
    const size_t off = (size_t)src * a.Dp;
    float post = 0.f;
    if (a.cout) {
        float ss = 0.f;
        for (int i = tid * 4; i < a.Dp; i += 1024) {
            float4 y = *reinterpret_cast<const float4 *>(a.cout + off + i);
            if (a.post_b) {
                const float4 b = *reinterpret_cast<const float4 *>(a.post_b + i);
                y.x += b.x; y.y += b.y; y.z += b.z; y.w += b.w;
            }
            *reinterpret_cast<float4 *>(row + i) = y;     // (the weight's padding rows are zero)
            ss += (y.x * y.x + y.y * y.y) + (y.z * y.z + y.w * y.w);
        }
        post = 1.f / sqrtf(block_sum(ss, sm) / (float)a.D + a.eps);
    }
    float ss = 0.f, mx = 0.f;
    for (int i = tid * 4; i < a.Dp; i += 1024) {          // the thread's own entries
        float4 v = *reinterpret_cast<const float4 *>(a.x + off + i);
        const float4 g = *reinterpret_cast<const float4 *>(a.g + i);
        if (a.cout) {
            const float4 y = *reinterpret_cast<const float4 *>(row + i), w = *reinterpret_cast<const float4 *>(a.post_g + i);
            v.x = fmaf(y.x * post, w.x, v.x); v.y = fmaf(y.y * post, w.y, v.y); v.z = fmaf(y.z * post, w.z, v.z); v.w = fmaf(y.w * post, w.w, v.w);
            if (a.keep) *reinterpret_cast<float4 *>(a.x + off + i) = v;
        }
        ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
        const float4 h = make_float4(v.x * g.x, v.y * g.y, v.z * g.z, v.w * g.w);
        *reinterpret_cast<float4 *>(row + i) = h;
        mx = fmaxf(mx, fmaxf(fmaxf(fabsf(h.x), fabsf(h.y)), fmaxf(fabsf(h.z), fabsf(h.w))));
    }
    block_sum_max(ss, mx, sm);                            // its barriers also publish the row
    const float inv = 1.f / sqrtf(ss / (float)a.D + a.eps);
    if (a.h)
        for (int i = tid; i < a.Dp; i += 256) a.h[(size_t)m * a.Dp + i] = row[i] * inv;
    if (a.a16) {
        const float s = row_scale_for(mx * inv);
        store_row_f16(row, a.Dp, a.a16, m, tiled_kb(a.Dp), s * inv);
        if (tid == 0) a.inv[m] = 1.f / s;
    }
}

// One workgroup of NT threads per row.  A thread holds P pieces of eight columns in registers; what a row has beyond them is
// formed twice.
template <int NT, int P>
__global__ __launch_bounds__(NT) void k_gelu_rows(ActRows a)
{
    __shared__ float sm[16];
    const int m = xcd_block_row(blockIdx.x, gridDim.x), tid = threadIdx.x;
    const float *up = a.up + (size_t)m * a.ld;
    auto ask = [&](int k, float4 (&p)[2]) __attribute__((always_inline)) {
#pragma unroll
        for (int e = 0; e < 2; e++) p[e] = k < a.K ? *reinterpret_cast<const float4 *>(up + k + 4 * e) : make_float4(0.f, 0.f, 0.f, 0.f);
    };
    auto act = [&](int k, float4 (&p)[2]) __attribute__((always_inline)) {
        float mx = 0.f;
#pragma unroll
        for (int e = 0; e < 8; e++) {
            float &v = (&p[e >> 2].x)[e & 3];
            v = k + e < a.n ? gelu_tanh(v) : 0.f;
            mx = fmaxf(mx, fabsf(v));
        }
        return mx;
    };
    const int Kb = tiled_kb(a.K);
    auto put = [&](int k, const float4 (&p)[2], float s) __attribute__((always_inline)) {
        half8 h;
#pragma unroll
        for (int e = 0; e < 8; e++) h[e] = f2h((&p[e >> 2].x)[e & 3] * s);
        if (k < Kb * 64) *reinterpret_cast<half8 *>(&a.a16[tiled_a_index(m, k, Kb)]) = h;
    };
    float4 v[P][2], x[2];
    float mx = 0.f;
#pragma unroll
    for (int i = 0; i < P; i++) ask((i * NT + tid) * 8, v[i]);
#pragma unroll
    for (int i = 0; i < P; i++) mx = fmaxf(mx, act((i * NT + tid) * 8, v[i]));
    for (int k = (P * NT + tid) * 8; k < a.K; k += NT * 8) { ask(k, x); mx = fmaxf(mx, act(k, x)); }
    const float s = row_scale_for(block_max(mx, sm));
#pragma unroll
    for (int i = 0; i < P; i++) put((i * NT + tid) * 8, v[i], s);
    for (int k = (P * NT + tid) * 8; k < Kb * 64; k += NT * 8) { ask(k, x); act(k, x); put(k, x, s); }
    if (tid == 0) a.inv[m] = 1.f / s;
}

__global__ __launch_bounds__(256) void k_gelu_rows_f32(ActRows a)
{
    const size_t m = blockIdx.x;
    for (int i = threadIdx.x; i < a.K; i += 256) a.h[m * a.K + i] = i < a.n ? gelu_tanh_exact(a.up[m * a.ld + i]) : 0.f;
}

__global__ __launch_bounds__(256) void k_rope_table(float2 *tab, int n, int pairs, const double *__restrict__ freq)
{
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const double angle = (double)(i / pairs) * freq[i % pairs];
    tab[i] = make_float2((float)cos(angle), (float)sin(angle));
}

}  // namespace

void launch_norms_around(const AroundRows &a, int rows) { LAUNCH(k_norms_around, dim3(rows), dim3(256), (size_t)a.Dp * 4, a); }

void launch_gelu_rows(const ActRows &a, int rows)
{
    if (a.h) LAUNCH(k_gelu_rows_f32, dim3(rows), dim3(256), 0, a);
    else if (a.K <= 4096) LAUNCH((k_gelu_rows<256, 2>), dim3(rows), dim3(256), 0, a);
    else LAUNCH((k_gelu_rows<512, 4>), dim3(rows), dim3(512), 0, a);
}

void launch_rope_table(float2 *tab, int max_seq, const std::vector<double> &freqs)
{
    const int pairs = (int)freqs.size(), n = max_seq * pairs;
    if (n <= 0) return;
    MetalBuf *f = metal_buf_from_data(freqs.data(), freqs.size() * sizeof(double));
    LAUNCH(k_rope_table, dim3((n + 255) / 256), dim3(256), 0, tab, n, pairs, dptr_as<double>(f));
    metal_buf_free(f);                                    // synchronises the stream first
}

void launch_embed_rows(const float *emb, const int *tok, float scale, float *x, int D, int Dp, int rows)
{
    LAUNCH(k_embed_rows, dim3((Dp + 255) / 256, rows), dim3(256), 0, emb, tok, scale, x, D, Dp);
}

void launch_embed_few(const float *emb, const int *tok, float scale, float *x, int D, int Dp, int rows)
{
    FewTokens t{};
    for (int i = 0; i < rows; i++) t.id[i] = tok[i];
    LAUNCH(k_embed_few, dim3((Dp + 255) / 256, rows), dim3(256), 0, emb, t, scale, x, D, Dp);
}

void launch_norm_rows(const NormRows &a, int rows) { LAUNCH(k_norm_rows, dim3(rows), dim3(256), (size_t)a.Dp * 4, a); }

}  // namespace lmhip
