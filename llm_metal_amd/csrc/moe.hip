// Mixture of experts: softmax router with the largest scores chosen, squared-ReLU experts.
#include "stack.h"
#include "expert.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

// One wave per row: its experts and their weights
__global__ __launch_bounds__(256) void k_route(MoeRows a)
{
    const int m = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (m >= a.rows) return;
    route_row(a.z + (size_t)m * a.ldz, a.E, a.top, lane, a.idx + (size_t)m * a.top, a.w + (size_t)m * a.top);
}

// act[m][s][i] = relu(up_e[i] . h[m])^2 for the s-th chosen expert e of row m; a wave per i.  grid (ceil(ffp / 4), top, rows)
template <typename WT>
__global__ __launch_bounds__(256) void k_expert_up(MoeRows a)
{
    const int lane = threadIdx.x & 63, i = blockIdx.x * 4 + (threadIdx.x >> 6), s = blockIdx.y, m = blockIdx.z;
    if (i >= a.ffp) return;
    const size_t slot = (size_t)m * a.top + s;
    float v = 0.f;
    if (i < a.ff) v = wave_sum(dot_part((const WT *)a.up + ((size_t)a.idx[slot] * a.up_rows + i) * a.Dp, a.h + (size_t)m * a.Dp, a.Dp, lane));
    if (lane == 0) a.act[slot * a.ffp + i] = relu2(v);   // the padding is written too: zero
}

// y[m][d] = sum over the chosen experts of w * (down_e[d] . act); a wave per d.  grid (ceil(Dp / 4), rows)
template <typename WT>
__global__ __launch_bounds__(256) void k_expert_down(MoeRows a)
{
    const int lane = threadIdx.x & 63, d = blockIdx.x * 4 + (threadIdx.x >> 6), m = blockIdx.y;
    if (d >= a.Dp) return;
    float y = 0.f;
    if (d < a.D)
        for (int s = 0; s < a.top; s++) {
            const size_t slot = (size_t)m * a.top + s;
            y = fmaf(a.w[slot], dot_part((const WT *)a.down + ((size_t)a.idx[slot] * a.down_rows + d) * a.ffp, a.act + slot * a.ffp, a.ffp, lane), y);
        }
    y = wave_sum(y);
    if (lane == 0) a.y[(size_t)m * a.Dp + d] = y;
}

// ---------------------------------------------------------------- pairs sorted by expert

// grid (E), block 256: how many pairs chose expert blockIdx.x
__global__ __launch_bounds__(256) void k_moe_count(const int *__restrict__ idx, int n, int *__restrict__ count)
{
    __shared__ float sm[16];
    int c = 0;
#pragma unroll 8
    for (int i = threadIdx.x; i < n; i += 256) c += idx[i] == (int)blockIdx.x;
    const float total = block_sum((float)c, sm);          // exact: far below 2^24
    if (threadIdx.x == 0) count[blockIdx.x] = (int)total;
}

// grid (E), block 256: the expert's blocks, and its pairs in order of row into them
__global__ __launch_bounds__(256) void k_moe_place(const int *__restrict__ idx, int n, int top, int E, MoeGroups g)
{
    __shared__ float sm[16];
    __shared__ int wave_n[4];
    const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    int before = 0;                                       // blocks of the experts ahead
    for (int i = tid; i < e; i += 256) before += (g.count[i] + 127) >> 7;
    const int t0 = (int)block_sum((float)before, sm), mine = g.count[e], nt = (mine + 127) >> 7;
    for (int i = tid; i < nt; i += 256) g.of[t0 + i] = e;
    for (int i = mine + tid; i < nt * 128; i += 256) g.src[t0 * 128 + i] = -1;
    if (e == E - 1 && tid == 0) g.of[g.tiles] = t0 + nt;
    if (e == E - 1)                                       // blocks behind the last expert's
        for (int i = t0 + nt + tid; i < g.tiles; i += 256) g.of[i] = -1;
    if (!mine) return;
    int at = t0 * 128;
    constexpr int U = 8;                                  // 256 U pairs per trip, their reads in flight together
    for (int i0 = 0; i0 < n; i0 += 256 * U) {
        bool hit[U];
        int rank[U], in_wave = 0;
#pragma unroll
        for (int u = 0; u < U; u++) { const int i = i0 + (wave * U + u) * 64 + lane; hit[u] = i < n && idx[min(i, n - 1)] == e; }
#pragma unroll
        for (int u = 0; u < U; u++) {
            const unsigned long long b = __ballot(hit[u]);
            rank[u] = in_wave + __popcll(b & ((1ull << lane) - 1ull));
            in_wave += __popcll(b);
        }
        if (lane == 0) wave_n[wave] = in_wave;
        __syncthreads();
        int o = at;
        for (int w = 0; w < wave; w++) o += wave_n[w];
#pragma unroll
        for (int u = 0; u < U; u++)
            if (hit[u]) {
                const int i = i0 + (wave * U + u) * 64 + lane;
                g.src[o + rank[u]] = i / top;
                g.pos[i] = o + rank[u];
            }
        at += wave_n[0] + wave_n[1] + wave_n[2] + wave_n[3];
        __syncthreads();
    }
}

// grid (row blocks of 32, chunks of K blocks), block 256: rows of a tiled operand to other places.  A wave writes whole 1 KB
// slices; a row is 32 contiguous bytes of its source slice.
__global__ __launch_bounds__(256) void k_moe_gather(MoeGroups g, const half_t *__restrict__ a16, const float *__restrict__ inv,
                                                    half_t *__restrict__ out16, float *__restrict__ out_inv, int Kb, int per)
{
    const int rb = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (g.of[rb >> 2] < 0) return;
    const int m = g.src[rb * 32 + (lane >> 1)], src = max(m, 0);
    const half8 *from = reinterpret_cast<const half8 *>(a16) + ((size_t)(src >> 5) * Kb) * 256 + ((src & 31) << 1) + (lane & 1);
    half8 *to = reinterpret_cast<half8 *>(out16) + (size_t)rb * Kb * 256 + lane;
    const int s0 = blockIdx.y * per * 4, s1 = min(s0 + per * 4, Kb * 4);
    for (int s = s0 + wave; s < s1; s += 4 * 4) {         // four slices of a wave in flight
        half8 v[4];
#pragma unroll
        for (int u = 0; u < 4; u++) v[u] = from[(size_t)min(s + 4 * u, s1 - 1) * 64];
#pragma unroll
        for (int u = 0; u < 4; u++) if (s + 4 * u < s1) to[(size_t)(s + 4 * u) * 64] = v[u];
    }
    if (blockIdx.y == 0 && threadIdx.x < 32) { const int r = g.src[rb * 32 + threadIdx.x]; if (r >= 0) out_inv[rb * 32 + threadIdx.x] = inv[r]; }
}

// grid (rows of the groups), block 256
__global__ __launch_bounds__(256) void k_moe_act(MoeGroups g, const float *__restrict__ up, int ld, int n, half_t *__restrict__ out16,
                                                 float *__restrict__ out_inv, int K)
{
    extern __shared__ float row[];                        // [K]
    __shared__ float sm[16];
    const int p = blockIdx.x;
    if (g.of[p >> 7] < 0 || g.src[p] < 0) return;
    float mx = 0.f;
    for (int i = threadIdx.x; i < K; i += 256) {
        const float v = i < n ? relu2(up[(size_t)p * ld + i]) : 0.f;
        row[i] = v;
        mx = fmaxf(mx, v);
    }
    const float s = row_scale_for(block_max(mx, sm));     // its barriers publish the row
    store_row_f16(row, K, out16, p, tiled_kb(K), s);
    if (threadIdx.x == 0) out_inv[p] = 1.f / s;
}

}  // namespace

int moe_group_tiles(int rows, int top, int E) { const int n = rows * top; return n / 128 + (E < n ? E : n); }
size_t moe_group_ints(int rows, int top, int E) { const size_t t = moe_group_tiles(rows, top, E); return (size_t)E + t + 1 + t * 128 + (size_t)rows * top; }
MoeGroups moe_groups_at(int *base, int rows, int top, int E)
{
    MoeGroups g{};
    g.tiles = moe_group_tiles(rows, top, E);
    g.count = base; g.of = g.count + E; g.src = g.of + g.tiles + 1; g.pos = g.src + (size_t)g.tiles * 128;
    return g;
}

void launch_moe_groups(const MoeRows &a, const MoeGroups &g)
{
    const int n = a.rows * a.top;
    LAUNCH(k_moe_count, dim3(a.E), dim3(256), 0, a.idx, n, g.count);
    LAUNCH(k_moe_place, dim3(a.E), dim3(256), 0, a.idx, n, a.top, a.E, g);
}

void launch_moe_gather(const MoeGroups &g, const half_t *a16, const float *inv, half_t *out16, float *out_inv, int K)
{
    const int Kb = tiled_kb(K), per = 16;
    LAUNCH(k_moe_gather, dim3(g.tiles * 4, (Kb + per - 1) / per), dim3(256), 0, g, a16, inv, out16, out_inv, Kb, per);
}

void launch_moe_act(const MoeGroups &g, const float *up, int ld, int n, half_t *out16, float *out_inv, int K)
{
    LAUNCH(k_moe_act, dim3(g.tiles * 128), dim3(256), (size_t)K * 4, g, up, ld, n, out16, out_inv, K);
}

void launch_route(const MoeRows &a) { LAUNCH(k_route, dim3((a.rows + 3) / 4), dim3(256), 0, a); }

void launch_experts_per_row(const MoeRows &a)
{
    const dim3 up((a.ffp + 3) / 4, a.top, a.rows), down((a.Dp + 3) / 4, a.rows);
    if (a.f32) { LAUNCH(k_expert_up<float>, up, dim3(256), 0, a); LAUNCH(k_expert_down<float>, down, dim3(256), 0, a); }
    else { LAUNCH(k_expert_up<half_t>, up, dim3(256), 0, a); LAUNCH(k_expert_down<half_t>, down, dim3(256), 0, a); }
}

}  // namespace lmhip
