// Merge of split decode attention: every (token, head) has NP partitions of its keys, each with an
// unnormalised weighted sum of values, its maximum (log2 units) and its sum of weights.
//   o = out_scale * sum_p 2^(m_p - M) part_p / (sum_p 2^(m_p - M) l_p [+ exp(sink_h) 2^-M])
#include "rt_paged.h"

namespace rt {

constexpr int MERGE_MAX = 1024;  // partitions

// one workgroup per (token, head); an empty partition has m = -inf, l = 0 and no part
__global__ __launch_bounds__(128) void partition_merge_kernel(const float* __restrict__ part, const float* __restrict__ ml,
                                                              const float* __restrict__ sink, bf16_t* __restrict__ o,
                                                              long ldo, int H, int rank, int NP, float out_scale) {
  __shared__ float fac[MERGE_MAX];
  __shared__ float sbuf[2];
  const long th = blockIdx.x;
  const int tid = threadIdx.x, h = (int)(th % H);
  const float sink2 = sink ? sink[h] * 1.4426950408889634f : -INFINITY;
  const float* m = ml + th * NP * 2;
  float mx = -INFINITY;
  for (int p = tid; p < NP; p += 128) {
    fac[p] = m[2 * p];
    mx = fmaxf(mx, fac[p]);
  }
  const float M = fmaxf(block_max(mx, sbuf), sink2);
  float L = 0.f;
  for (int p = tid; p < NP; p += 128) {
    fac[p] = exp2f(fac[p] - M);  // 0 for an empty partition
    L += m[2 * p + 1] * fac[p];
  }
  const float inv = out_scale / (block_sum(L, sbuf) + exp2f(sink2 - M));
  bf16_t* od = o + th / H * ldo + (long)h * rank;
  for (int c = 4 * tid; c < rank; c += 512) {  // rank % 8 == 0
    float y[4] = {0.f, 0.f, 0.f, 0.f};
    for (int p0 = 0; p0 < NP; p0 += 8) {  // eight partitions' rows in flight
      float4 v[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = *(const float4*)(part + (th * NP + min(p0 + j, NP - 1)) * rank + c);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float f = p0 + j < NP ? fac[p0 + j] : 0.f;
        if (f != 0.f) {  // an empty partition wrote nothing
          y[0] = fmaf(f, v[j].x, y[0]); y[1] = fmaf(f, v[j].y, y[1]);
          y[2] = fmaf(f, v[j].z, y[2]); y[3] = fmaf(f, v[j].w, y[3]);
        }
      }
    }
    *(uint2*)(od + c) = make_uint2(pack2bf(y[0] * inv, y[1] * inv), pack2bf(y[2] * inv, y[3] * inv));
  }
}

}  // namespace rt

using namespace rt;

// o [T, H * rank] bf16 with row stride ldo; rank % 8 == 0, ldo % 4 == 0
extern "C" int rt_partition_merge(const float* part, const float* ml, const float* sink, void* o, long ldo, int T, int H,
                                  int rank, int NP, float out_scale, hipStream_t stream) {
  if (T <= 0) return 0;
  if (rank % 8 || ldo % 4 || (uintptr_t)o % 8 || NP < 1 || NP > MERGE_MAX) return -1;
  hipLaunchKernelGGL(partition_merge_kernel, dim3((unsigned)((long)T * H)), dim3(128), 0, stream, part, ml, sink, (bf16_t*)o,
                     ldo, H, rank, NP, out_scale);
  RT_LAUNCH_CHECK();
  return 0;
}
