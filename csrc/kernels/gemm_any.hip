// GEMM without shape or type requirements: C = A W^T in fp32 arithmetic, A / W / C bf16 or fp32, any
// M, N, K and strides, optionally batched (one product per head) or grouped (one weight per expert
// over rows sorted by expert). It carries the fp32 mode of the models (true 32-bit: fp32 operands,
// v_fma_f32) and the bf16 sizes that the MFMA kernels of gemm_bf16.hip / gemm_big.hip do not take
// (K % 64 at few rows, K % 8, N % 8). 64x64 tile per workgroup, 4x4 outputs per thread, K-steps of 16
// through LDS as fp32 with the next step's loads in flight during the products.
//
// Also here: the elementwise steps of that path (gated linear unit, squared relu, output gate).
#include "rt_common.h"

namespace rt {

struct AnyArgs {
  const void* A; long lda, sA;   // A[b] = A + b * sA
  const void* W; long ldw, sW;
  void* C; long ldc, sC;
  int M, N, K;
  // grouped: rows [offs[g], offs[g + 1]) of C use weight g; row_map: A row behind each C row
  const int* offs; const int* row_map;
  int tiles_m;
};

template <typename T> __device__ __forceinline__ float any_ld(const T* p);
template <> __device__ __forceinline__ float any_ld<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float any_ld<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void any_st(T* p, float v);
template <> __device__ __forceinline__ void any_st<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void any_st<float>(float* p, float v) { *p = v; }

template <typename T, typename TC>
__global__ __launch_bounds__(256) void gemm_any_kernel(AnyArgs p) {
  constexpr int TM = 64, TN = 64, TK = 16, LD = 68;
  __shared__ __attribute__((aligned(16))) float As[TK][LD], Ws[TK][LD];
  const int b = blockIdx.z;
  int mbeg = 0, mend = p.M;
  if (p.offs) { mbeg = p.offs[b]; mend = p.offs[b + 1]; }
  const T* A = (const T*)p.A + (p.offs ? 0L : b * p.sA);
  const T* W = (const T*)p.W + b * p.sW;
  TC* C = (TC*)p.C + (p.offs ? 0L : b * p.sC);
  const int tid = threadIdx.x;
  const int n0 = blockIdx.x * TN;
  const int lr = tid >> 2, lk = (tid & 3) * 4;  // the thread's row and first k of a staged tile
  const int ty = tid >> 4, tx = tid & 15;
  for (int m0 = mbeg + blockIdx.y * TM; m0 < mend; m0 += gridDim.y * TM) {
    const int ar = m0 + lr, wr = n0 + lr;
    const bool a_ok = ar < mend, w_ok = wr < p.N;
    const T* ap = A + (long)(a_ok ? (p.row_map ? p.row_map[ar] : ar) : 0) * p.lda;
    const T* wp = W + (long)(w_ok ? wr : 0) * p.ldw;
    float acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;
    float ra[4], rw[4];
    auto load = [&](int k0) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int k = k0 + lk + e;
        ra[e] = a_ok && k < p.K ? any_ld(ap + k) : 0.f;
        rw[e] = w_ok && k < p.K ? any_ld(wp + k) : 0.f;
      }
    };
    load(0);
    for (int k0 = 0; k0 < p.K; k0 += TK) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        As[lk + e][lr] = ra[e];
        Ws[lk + e][lr] = rw[e];
      }
      __syncthreads();
      if (k0 + TK < p.K) load(k0 + TK);
#pragma unroll
      for (int k = 0; k < TK; ++k) {
        const float4 av = *(const float4*)&As[k][ty * 4], wv = *(const float4*)&Ws[k][tx * 4];
        const float a4[4] = {av.x, av.y, av.z, av.w}, w4[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a4[i], w4[j], acc[i][j]);
      }
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = m0 + ty * 4 + i;
      if (row >= mend) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int col = n0 + tx * 4 + j;
        if (col < p.N) any_st(C + (long)row * p.ldc + col, acc[i][j]);
      }
    }
  }
}

// gu [T, 2F] (gate | up) -> y [T, F]
template <typename T>
__global__ __launch_bounds__(256) void glu_any_kernel(const T* __restrict__ gu, long ldg, T* __restrict__ y, long n,
                                                      int F, GluP gp) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const long t = i / F;
  const int c = (int)(i % F);
  float g = any_ld(gu + t * ldg + c), u = any_ld(gu + t * ldg + F + c);
  g = g > gp.limit ? gp.limit : g;
  u = u > gp.limit ? gp.limit : (u < -gp.limit ? -gp.limit : u);
  any_st(y + i, g / (1.f + expf(-(gp.alpha * g))) * (u + gp.offset));
}

// y = max(x, 0)^2 of an fp32 product (act 8), or a rounding copy (act 0)
template <typename T>
__global__ __launch_bounds__(256) void act_any_kernel(const float* __restrict__ x, T* __restrict__ y, long n, int act) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  float v = x[i];
  if (act == 8) {
    v = fmaxf(v, 0.f);
    v *= v;
  }
  any_st(y + i, v);
}

// a [T, N] *= sigmoid(g [T, N]) (output gate of an attention layer)
template <typename T>
__global__ __launch_bounds__(256) void gate_mul_kernel(T* __restrict__ a, const T* __restrict__ g, long ldg, long n,
                                                       int N) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const float x = any_ld(g + i / N * ldg + i % N);
  any_st(a + i, any_ld(a + i) / (1.f + expf(-x)));
}

}  // namespace rt

using namespace rt;

// f32: operands fp32 (else bf16); out_f32: C fp32 (else the operand type's). batch > 1: strided products.
// offs (device int [groups + 1]): grouped form, batch = groups, M = upper bound of all rows together.
extern "C" int rt_gemm_any(int f32, int out_f32, const void* A, long lda, long sA, const void* W, long ldw, long sW,
                           void* C, long ldc, long sC, int M, int N, int K, int batch, const int* offs,
                           const int* row_map, hipStream_t stream) {
  if (M <= 0 || N <= 0 || batch <= 0) return 0;
  if (K <= 0) return -1;
  AnyArgs p{A, lda, sA, W, ldw, sW, C, ldc, sC, M, N, K, offs, row_map, 0};
  const int tm = (M + 63) / 64;
  // grouped: a few row tiles per group, the kernel walks the rest (the group sizes are device data)
  dim3 grid((N + 63) / 64, offs ? min(tm, 8) : min(tm, 65535), batch), block(256);
  if (batch > 65535) return -2;
  if (f32) hipLaunchKernelGGL((gemm_any_kernel<float, float>), grid, block, 0, stream, p);
  else if (out_f32) hipLaunchKernelGGL((gemm_any_kernel<bf16_t, float>), grid, block, 0, stream, p);
  else hipLaunchKernelGGL((gemm_any_kernel<bf16_t, bf16_t>), grid, block, 0, stream, p);
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_glu_any(int f32, const void* gu, long ldg, void* y, long T, int F, const float* glu_p,
                          hipStream_t stream) {
  const long n = T * F;
  if (n <= 0) return 0;
  GluP gp;
  if (glu_p) { gp.limit = glu_p[0]; gp.alpha = glu_p[1]; gp.offset = glu_p[2]; }
  dim3 grid((unsigned)((n + 255) / 256)), block(256);
  if (f32) hipLaunchKernelGGL((glu_any_kernel<float>), grid, block, 0, stream, (const float*)gu, ldg, (float*)y, n, F, gp);
  else hipLaunchKernelGGL((glu_any_kernel<bf16_t>), grid, block, 0, stream, (const bf16_t*)gu, ldg, (bf16_t*)y, n, F, gp);
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_act_any(int f32, const float* x, void* y, long n, int act, hipStream_t stream) {
  if (n <= 0) return 0;
  if (act != 0 && act != 8) return -1;
  dim3 grid((unsigned)((n + 255) / 256)), block(256);
  if (f32) hipLaunchKernelGGL((act_any_kernel<float>), grid, block, 0, stream, x, (float*)y, n, act);
  else hipLaunchKernelGGL((act_any_kernel<bf16_t>), grid, block, 0, stream, x, (bf16_t*)y, n, act);
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_gate_mul(int f32, void* a, const void* g, long ldg, long T, int N, hipStream_t stream) {
  const long n = T * N;
  if (n <= 0) return 0;
  dim3 grid((unsigned)((n + 255) / 256)), block(256);
  if (f32) hipLaunchKernelGGL((gate_mul_kernel<float>), grid, block, 0, stream, (float*)a, (const float*)g, ldg, n, N);
  else hipLaunchKernelGGL((gate_mul_kernel<bf16_t>), grid, block, 0, stream, (bf16_t*)a, (const bf16_t*)g, ldg, n, N);
  RT_LAUNCH_CHECK();
  return 0;
}
