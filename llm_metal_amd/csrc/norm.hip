// The residual row kernels of a layer-by-layer model: embedding rows, and the residual sum with the layer norm that
// feeds a product.
#include "stack.h"
#include "rows.h"

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

}  // namespace

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
