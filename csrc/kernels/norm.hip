// Normalisation kernels: fused residual-add + RMSNorm (decoder) and fused
// residual-add + LayerNorm (encoders / OPT), forward and backward.
//
// Forward contract (both norms):
//   h = x (+ res)            -> written to h_out when res is given (the new residual stream)
//   y = norm(h) * w (+ b)    -> bf16
//   rstd (and mean for LN)   -> fp32 per row (saved for backward)
// One workgroup per row; the row lives in registers (16-B vectors, <= 8 per thread), so a row is
// read once and written once: the op runs at the HBM roofline. Reductions are wave64 shuffles
// followed by one LDS exchange.
#include "rt_common.h"

namespace rt {

constexpr int NORM_MAXV = 8;  // max 16-B vectors per thread -> H <= 256*8*8 = 16384

template <bool LAYERNORM, int NV, int MAXT = 512>
__global__ __launch_bounds__(MAXT) void norm_fwd_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ res,
                                                       const bf16_t* __restrict__ w, const bf16_t* __restrict__ b,
                                                       bf16_t* __restrict__ y, bf16_t* __restrict__ h_out,
                                                       float* __restrict__ rstd_out, float* __restrict__ mean_out,
                                                       int H, float eps, const float* __restrict__ xs, int nsplit,
                                                       long sstride) {
  // xs != null: x is the bf16-rounded sum of nsplit fp32 split-K slabs (stride sstride floats):
  // the split-K reduce of the producing GEMM fused into this pass (decode at batch 65..512)
  __shared__ float sbuf[16];  // <= 16 waves
  const long row = blockIdx.x;
  const int nv = H / 8;
  const bf16_t* xr = x + row * H;
  float v[NV][8];
  float s = 0.f;
  // weight (and bias) loads are issued with the row loads: one memory round trip before the
  // reduction instead of a second dependent one after it (decode rows are latency-bound)
  uint4 wraw[NV], braw[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nv) {
      wraw[i] = *(const uint4*)(w + c * 8);
      if (LAYERNORM && b) braw[i] = *(const uint4*)(b + c * 8);
    }
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nv) {
      if (xs) {
        float t8[8];
        sum_slabs8(xs + row * H + c * 8, sstride, nsplit, t8);
#pragma unroll
        for (int k = 0; k < 8; ++k) v[i][k] = bf2f(f2bf(t8[k]));  // = the reduce kernel's bf16 output
      } else {
        unpack8(*(const uint4*)(xr + c * 8), v[i]);
      }
      if (res) {
        float r[8];
        unpack8(*(const uint4*)(res + row * H + c * 8), r);
#pragma unroll
        for (int k = 0; k < 8; ++k) v[i][k] += r[k];
        // the residual stream is kept in bf16: round before normalising so fwd == what bwd sees
#pragma unroll
        for (int k = 0; k < 8; ++k) v[i][k] = bf2f(f2bf(v[i][k]));
        *(uint4*)(h_out + row * H + c * 8) = pack8(v[i]);
      }
#pragma unroll
      for (int k = 0; k < 8; ++k) s += LAYERNORM ? v[i][k] : v[i][k] * v[i][k];
    }
  }
  float mean = 0.f, rstd;
  if (LAYERNORM) {
    mean = block_sum(s, sbuf) / H;
    float s2 = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nv)
#pragma unroll
        for (int k = 0; k < 8; ++k) { const float d = v[i][k] - mean; s2 += d * d; }
    }
    rstd = rsqrtf(block_sum(s2, sbuf) / H + eps);
  } else {
    rstd = rsqrtf(block_sum(s, sbuf) / H + eps);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < nv) {
      float wv[8], bv[8], o[8];
      unpack8(wraw[i], wv);
      if (LAYERNORM && b) unpack8(braw[i], bv);
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        o[k] = (v[i][k] - mean) * rstd * wv[k];
        if (LAYERNORM && b) o[k] += bv[k];
      }
      *(uint4*)(y + row * H + c * 8) = pack8(o);
    }
  }
  if (threadIdx.x == 0) {
    if (rstd_out) rstd_out[row] = rstd;
    if (LAYERNORM && mean_out) mean_out[row] = mean;
  }
}

// Backward. Each workgroup walks `rows_per_block` rows, accumulating dw (and db) in registers,
// then stores its partial as row blockIdx.x of the fp32 dw / db slabs [gridDim.x, H] (the caller
// sums the rows in a fixed order: no arrival-order atomics).
//   xhat = (h - mean) * rstd ; y = xhat*w (+b)
//   g = dy*w ; dh = rstd * (g - mean(g) [LN only] - xhat * mean(g*xhat))  (+ dh_res)
template <bool LAYERNORM, int NV>
__global__ __launch_bounds__(256) void norm_bwd_kernel(const bf16_t* __restrict__ dy, const bf16_t* __restrict__ h,
                                                       const bf16_t* __restrict__ w, const float* __restrict__ rstd_in,
                                                       const float* __restrict__ mean_in,
                                                       const bf16_t* __restrict__ dh_res, bf16_t* __restrict__ dh,
                                                       float* __restrict__ dw, float* __restrict__ db, int T, int H,
                                                       int rows_per_block) {
  __shared__ float sbuf[8];
  const int nv = H / 8;
  float dwacc[NV][8], dbacc[NV][8];
  float wv[NV][8];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
#pragma unroll
    for (int k = 0; k < 8; ++k) { dwacc[i][k] = 0.f; dbacc[i][k] = 0.f; }
    if (c < nv) unpack8(*(const uint4*)(w + c * 8), wv[i]);
  }
  const long r0 = (long)blockIdx.x * rows_per_block;
  for (long row = r0; row < min((long)T, r0 + rows_per_block); ++row) {
    const float rstd = rstd_in[row];
    const float mean = LAYERNORM ? mean_in[row] : 0.f;
    float xh[NV][8], gg[NV][8];
    float s_g = 0.f, s_gx = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nv) {
        float hv[8], dv[8];
        unpack8(*(const uint4*)(h + row * H + c * 8), hv);
        unpack8(*(const uint4*)(dy + row * H + c * 8), dv);
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          xh[i][k] = (hv[k] - mean) * rstd;
          gg[i][k] = dv[k] * wv[i][k];
          s_g += gg[i][k];
          s_gx += gg[i][k] * xh[i][k];
          dwacc[i][k] += dv[k] * xh[i][k];
          dbacc[i][k] += dv[k];
        }
      }
    }
    const float mg = LAYERNORM ? block_sum(s_g, sbuf) / H : 0.f;
    const float mgx = block_sum(s_gx, sbuf) / H;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nv) {
        float o[8], rr[8];
        if (dh_res) unpack8(*(const uint4*)(dh_res + row * H + c * 8), rr);
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          o[k] = rstd * (gg[i][k] - mg - xh[i][k] * mgx);
          if (dh_res) o[k] += rr[k];
        }
        *(uint4*)(dh + row * H + c * 8) = pack8(o);
      }
    }
  }
  if (dw || db) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nv)
#pragma unroll
        for (int k = 0; k < 8; ++k) {
          if (dw) dw[(long)blockIdx.x * H + c * 8 + k] = dwacc[i][k];
          if (LAYERNORM && db) db[(long)blockIdx.x * H + c * 8 + k] = dbacc[i][k];
        }
    }
  }
}

static void norm_geom(int H, int& threads, int& nvpt) {
  const int nv = H / 8;
  threads = nv >= 256 ? 256 : ((nv + 63) / 64) * 64;
  const int need = (nv + threads - 1) / threads;
  nvpt = need <= 1 ? 1 : need <= 2 ? 2 : need <= 4 ? 4 : 8;
}

}  // namespace rt

using namespace rt;

#define NORM_DISPATCH(LN, KER, ...)                                                              \
  switch (nvpt) {                                                                                \
    case 1: hipLaunchKernelGGL((KER<LN, 1>), __VA_ARGS__); break;                                 \
    case 2: hipLaunchKernelGGL((KER<LN, 2>), __VA_ARGS__); break;                                 \
    case 4: hipLaunchKernelGGL((KER<LN, 4>), __VA_ARGS__); break;                                 \
    default: hipLaunchKernelGGL((KER<LN, 8>), __VA_ARGS__); break;                                \
  }

extern "C" int rt_norm_fwd(int layernorm, const void* x, const void* res, const void* w, const void* b, void* y,
                           void* h_out, float* rstd, float* mean, int T, int H, float eps, const float* xs,
                           int nsplit, hipStream_t stream) {
  if (H % 8 != 0 || H > 256 * 8 * NORM_MAXV) return -1;
  if (T == 0) return 0;
  int threads, nvpt;
  norm_geom(H, threads, nvpt);
  // split-K slab reduce (decode at batch 65..512: one row per block, rows <= CUs): twice the waves
  // per row (one 8-element chunk per thread) keep twice the slab loads in flight per CU
  const int sl = tuning().norm_slab_threads;
  if (xs && sl >= 512 && H / 8 >= 512 && H / 8 <= 512) {
    threads = 512;
    nvpt = 1;
  }
  // H = 5120 (Llama-2-13B, config 5): one chunk per thread over 640 threads — the 256-thread form
  // sums three chunks' slabs one memory round trip after another (19.6 us per norm at batch 256)
  if (xs && sl >= 512 && H / 8 > 512 && H / 8 <= 1024) {
    const int t = (H / 8 + 63) / 64 * 64;
    if (layernorm)
      hipLaunchKernelGGL((norm_fwd_kernel<true, 1, 1024>), dim3(T), dim3(t), 0, stream, (const bf16_t*)x,
                         (const bf16_t*)res, (const bf16_t*)w, (const bf16_t*)b, (bf16_t*)y, (bf16_t*)h_out, rstd, mean,
                         H, eps, xs, nsplit, (long)T * H);
    else
      hipLaunchKernelGGL((norm_fwd_kernel<false, 1, 1024>), dim3(T), dim3(t), 0, stream, (const bf16_t*)x,
                         (const bf16_t*)res, (const bf16_t*)w, (const bf16_t*)b, (bf16_t*)y, (bf16_t*)h_out, rstd, mean,
                         H, eps, xs, nsplit, (long)T * H);
    RT_LAUNCH_CHECK();
    return 0;
  }
  if (layernorm) {
    NORM_DISPATCH(true, norm_fwd_kernel, dim3(T), dim3(threads), 0, stream, (const bf16_t*)x, (const bf16_t*)res,
                  (const bf16_t*)w, (const bf16_t*)b, (bf16_t*)y, (bf16_t*)h_out, rstd, mean, H, eps, xs, nsplit,
                  (long)T * H)
  } else {
    NORM_DISPATCH(false, norm_fwd_kernel, dim3(T), dim3(threads), 0, stream, (const bf16_t*)x, (const bf16_t*)res,
                  (const bf16_t*)w, (const bf16_t*)b, (bf16_t*)y, (bf16_t*)h_out, rstd, mean, H, eps, xs, nsplit,
                  (long)T * H)
  }
  RT_LAUNCH_CHECK();
  return 0;
}

// workgroups of rt_norm_bwd for T rows (= the rows of its dw / db partial slabs)
extern "C" int rt_norm_bwd_blocks(int T) {
  if (T <= 0) return 0;
  const int nblk = T < 1024 ? T : 1024;
  const int rpb = (T + nblk - 1) / nblk;
  return (T + rpb - 1) / rpb;
}

// dw / db (optional): fp32 [rt_norm_bwd_blocks(T), H] partial slabs, every row written
extern "C" int rt_norm_bwd(int layernorm, const void* dy, const void* h, const void* w, const float* rstd,
                           const float* mean, const void* dh_res, void* dh, float* dw, float* db, int T, int H,
                           hipStream_t stream) {
  if (H % 8 != 0 || H > 256 * 8 * NORM_MAXV) return -1;
  if (T == 0) return 0;
  int threads, nvpt;
  norm_geom(H, threads, nvpt);
  const int nblk = T < 1024 ? T : 1024;
  const int rpb = (T + nblk - 1) / nblk;
  const int grid = rt_norm_bwd_blocks(T);
  if (layernorm) {
    NORM_DISPATCH(true, norm_bwd_kernel, dim3(grid), dim3(threads), 0, stream, (const bf16_t*)dy, (const bf16_t*)h,
                  (const bf16_t*)w, rstd, mean, (const bf16_t*)dh_res, (bf16_t*)dh, dw, db, T, H, rpb)
  } else {
    NORM_DISPATCH(false, norm_bwd_kernel, dim3(grid), dim3(threads), 0, stream, (const bf16_t*)dy, (const bf16_t*)h,
                  (const bf16_t*)w, rstd, mean, (const bf16_t*)dh_res, (bf16_t*)dh, dw, db, T, H, rpb)
  }
  RT_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------------------
// Branch norm: the step between two sublayers of a decoder with a norm after each, and maybe one before
// (fp32 residual stream x [T, H], everything in fp32):
//   x += rms(y) * w_branch [* scale]     (y = the sublayer's output)
//   h  = rms(x) * w_next * next_mul      (the next sublayer's input, rounded once to the activation type)
//   h  = x                               (w_next == null: sublayers that read the stream itself)
// One workgroup per row, the row in registers: x is read and written once, y read once. The branch y is
//   Y_NONE    absent (first norm of a pass): x = table[ids[row]] when a table is given, normed and weighted
//             with w_branch if there is one;
//   Y_ACT     rows of the activation type;
//   Y_SLABS   the sum of nsplit fp32 slabs (split-K partial products; 1 slab = an fp32 tensor);
//   Y_PAIRS   a mixture: sum over the row's K slots of pair_w[row, k] * y[pair_pos[row, k]].
// h == null: x only.
// ---------------------------------------------------------------------------------------------
namespace rt {

enum BranchKind { Y_NONE = 0, Y_ACT = 1, Y_SLABS = 2, Y_PAIRS = 3, Y_PAIRS_F32 = 4 };

struct BranchArgs {
  float* x;
  const void* y; long y_stride; int nsplit;  // Y_SLABS: slab stride in floats
  const void* w_branch; const void* scale; const void* w_next; float next_mul; void* h;
  const void* table; const long* ids; int vocab;
  const float* pair_w; const int* pair_pos; int K;
  int H;
  float eps;
};

template <typename T> __device__ __forceinline__ float act_ld(const T* p);
template <> __device__ __forceinline__ float act_ld<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float act_ld<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void act_st(T* p, float v);
template <> __device__ __forceinline__ void act_st<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void act_st<float>(float* p, float v) { *p = v; }

template <typename T, int V>
__device__ __forceinline__ void act_ldv(const T* p, float* o) {
  if constexpr (V == 4 && sizeof(T) == 2) {
    const uint2 v = *(const uint2*)p;
    o[0] = __uint_as_float(v.x << 16); o[1] = __uint_as_float(v.x & 0xffff0000u);
    o[2] = __uint_as_float(v.y << 16); o[3] = __uint_as_float(v.y & 0xffff0000u);
  } else if constexpr (V == 4) {
    const float4 v = *(const float4*)p;
    o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
  } else {
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = act_ld(p + e);
  }
}
template <typename T, int V>
__device__ __forceinline__ void act_stv(T* p, const float* o) {
  if constexpr (V == 4 && sizeof(T) == 2) *(uint2*)p = make_uint2(pack2bf(o[0], o[1]), pack2bf(o[2], o[3]));
  else if constexpr (V == 4) *(float4*)p = make_float4(o[0], o[1], o[2], o[3]);
  else {
#pragma unroll
    for (int e = 0; e < V; ++e) act_st(p + e, o[e]);
  }
}

// V elements per access (4, or 1 when H % 4 != 0), NV accesses per thread
template <typename T, int KIND, int V, int NV>
__global__ __launch_bounds__(512) void branch_norm_kernel(BranchArgs a) {
  __shared__ float sbuf[8];
  const long row = blockIdx.x;
  const int nvec = a.H / V;
  float* xr = a.x + row * a.H;
  float x[NV][V], y[NV][V];
  long tok = 0;
  if (KIND == Y_NONE && a.table) {
    tok = a.ids[row];
    tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
  }
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
#pragma unroll
    for (int e = 0; e < V; ++e) { x[i][e] = 0.f; y[i][e] = 0.f; }
    if (c >= nvec) continue;
    if (KIND == Y_NONE && a.table) act_ldv<T, V>((const T*)a.table + tok * a.H + c * V, x[i]);
    else act_ldv<float, V>(xr + c * V, x[i]);
    if constexpr (KIND == Y_ACT) {
      act_ldv<T, V>((const T*)a.y + row * a.H + c * V, y[i]);
    } else if constexpr (KIND == Y_SLABS) {
      for (int q = 0; q < a.nsplit; ++q) {
        float t[V];
        act_ldv<float, V>((const float*)a.y + q * a.y_stride + row * a.H + c * V, t);
#pragma unroll
        for (int e = 0; e < V; ++e) y[i][e] += t[e];
      }
    } else if constexpr (KIND == Y_PAIRS || KIND == Y_PAIRS_F32) {
      for (int k0 = 0; k0 < a.K; k0 += 4) {  // four pairs' rows in flight
        float w[4], t[4][V];
        long pr[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const long o = row * a.K + min(k0 + j, a.K - 1);
          w[j] = k0 + j < a.K ? a.pair_w[o] : 0.f;
          pr[j] = a.pair_pos[o];
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if constexpr (KIND == Y_PAIRS_F32) act_ldv<float, V>((const float*)a.y + pr[j] * a.H + c * V, t[j]);
          else act_ldv<T, V>((const T*)a.y + pr[j] * a.H + c * V, t[j]);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (k0 + j < a.K) {
#pragma unroll
            for (int e = 0; e < V; ++e) y[i][e] = fmaf(w[j], t[j][e], y[i][e]);
          }
      }
    }
#pragma unroll
    for (int e = 0; e < V; ++e) s += KIND == Y_NONE ? x[i][e] * x[i][e] : y[i][e] * y[i][e];
  }
  if (KIND == Y_NONE && a.table && a.w_branch) {
    const float rstd = 1.f / sqrtf(block_sum(s, sbuf) / a.H + a.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c >= nvec) continue;
      float w[V];
      act_ldv<T, V>((const T*)a.w_branch + c * V, w);
#pragma unroll
      for (int e = 0; e < V; ++e) x[i][e] *= rstd * w[e];
    }
  }
  if constexpr (KIND != Y_NONE) {
    const float rstd = 1.f / sqrtf(block_sum(s, sbuf) / a.H + a.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c >= nvec) continue;
      float w[V];
      act_ldv<T, V>((const T*)a.w_branch + c * V, w);
      if (a.scale) {
        float f[V];
        act_ldv<T, V>((const T*)a.scale + c * V, f);
#pragma unroll
        for (int e = 0; e < V; ++e) w[e] *= f[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) x[i][e] += y[i][e] * rstd * w[e];
    }
  }
  if (KIND != Y_NONE || a.table) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nvec) act_stv<float, V>(xr + c * V, x[i]);
    }
  }
  if (!a.h) return;
  if (!a.w_next) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = threadIdx.x + i * blockDim.x;
      if (c < nvec) act_stv<T, V>((T*)a.h + row * a.H + c * V, x[i]);
    }
    return;
  }
  s = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int e = 0; e < V; ++e) s += x[i][e] * x[i][e];
  const float rstd = a.next_mul / sqrtf(block_sum(s, sbuf) / a.H + a.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c >= nvec) continue;
    float w[V], o[V];
    act_ldv<T, V>((const T*)a.w_next + c * V, w);
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = x[i][e] * rstd * w[e];
    act_stv<T, V>((T*)a.h + row * a.H + c * V, o);
  }
}

template <typename T, int KIND>
static int launch_branch(const BranchArgs& a, int Tn, hipStream_t st) {
  const int V = a.H % 4 == 0 ? 4 : 1;
  const int nvec = a.H / V;
  int threads = 64;
  while (threads < 512 && threads * 2 < nvec) threads *= 2;
  const int per = (nvec + threads - 1) / threads;
#define BN_L(VV, NVV) hipLaunchKernelGGL((branch_norm_kernel<T, KIND, VV, NVV>), dim3(Tn), dim3(threads), 0, st, a)
  if (V == 4) {
    if (per <= 2) BN_L(4, 2);
    else if (per <= 4) BN_L(4, 4);
    else if (per <= 8) BN_L(4, 8);
    else return -2;
  } else {
    if (per <= 8) BN_L(1, 8);
    else if (per <= 32) BN_L(1, 32);
    else return -2;
  }
#undef BN_L
  return 0;
}

}  // namespace rt

extern "C" int rt_branch_norm(int f32, int kind, float* x, const void* y, long y_stride, int nsplit,
                              const void* w_branch, const void* scale, const void* w_next, float next_mul, void* h,
                              const void* table, const long* ids, int vocab, const float* pair_w, const int* pair_pos, int K, int T, int H, float eps,
                              hipStream_t stream) {
  if (T <= 0) return 0;
  rt::BranchArgs a{x, y, y_stride, nsplit, w_branch, scale, w_next, next_mul, h, table, ids, vocab, pair_w, pair_pos, K, H, eps};
  int rc = -1;
#define BK(KIND) rc = f32 ? rt::launch_branch<float, rt::KIND>(a, T, stream) : rt::launch_branch<rt::bf16_t, rt::KIND>(a, T, stream)
  switch (kind) {
    case rt::Y_NONE: BK(Y_NONE); break;
    case rt::Y_ACT: BK(Y_ACT); break;
    case rt::Y_SLABS: BK(Y_SLABS); break;
    case rt::Y_PAIRS: BK(Y_PAIRS); break;
    case rt::Y_PAIRS_F32: BK(Y_PAIRS_F32); break;
  }
#undef BK
  if (rc) return rc;
  RT_LAUNCH_CHECK();
  return 0;
}
