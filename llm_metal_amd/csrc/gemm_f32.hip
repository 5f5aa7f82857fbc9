// C[m][n] = sum_k A[m][k] W[n][k] with fp32 operands, products and sums: what a state in 32-bit precision multiplies
// with (the matrix cores' reduced-precision forms of fp32 are not used).
#include "stack.h"

namespace lmhip {
namespace {

constexpr int BT = 64, BK = 16, LD = BT + 4;

// a 64 x 64 block of C per workgroup of 256 threads, 4 x 4 of it per thread; operands through LDS, K major
__global__ __launch_bounds__(256) void k_gemm_f32(const float *__restrict__ A, int lda, const float *__restrict__ W, int ldw,
                                                  float *__restrict__ C, int ldc, int M, int N, int K)
{
    __shared__ float As[BK * LD], Ws[BK * LD];
    const int tid = threadIdx.x, m0 = blockIdx.y * BT, n0 = blockIdx.x * BT;
    const int tm = (tid >> 4) * 4, tn = (tid & 15) * 4;
    const int lr = tid >> 2, lk = (tid & 3) * 4;          // the thread's four K entries of one row of either operand
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += BK) {
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int k = k0 + lk + e;
            As[(lk + e) * LD + lr] = (m0 + lr < M && k < K) ? A[(size_t)(m0 + lr) * lda + k] : 0.f;
            Ws[(lk + e) * LD + lr] = (n0 + lr < N && k < K) ? W[(size_t)(n0 + lr) * ldw + k] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < BK; k++) {
            const float4 a = *reinterpret_cast<const float4 *>(&As[k * LD + tm]), w = *reinterpret_cast<const float4 *>(&Ws[k * LD + tn]);
            const float av[4] = {a.x, a.y, a.z, a.w}, wv[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i][j] = fmaf(av[i], wv[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < 4; j++)
            if (m0 + tm + i < M && n0 + tn + j < N) C[(size_t)(m0 + tm + i) * ldc + n0 + tn + j] = acc[i][j];
}

}  // namespace

void launch_gemm_f32(const float *A, int lda, const float *W, int ldw, float *C, int ldc, int M, int N, int K)
{
    if (M <= 0 || N <= 0) return;
    hipLaunchKernelGGL(k_gemm_f32, dim3((N + BT - 1) / BT, (M + BT - 1) / BT), dim3(256), 0, stream(), A, lda, W, ldw, C, ldc, M, N, K);
    HIP_CHECK(hipGetLastError());
}

}  // namespace lmhip
