// Shared by the attention kernels over paged caches (latent_attention.hip, window_attention.hip): pages of
// 64 tokens, element access by type, MFMA operand packing, LDS tile images, segments of a ragged batch.
#pragma once
#include "rt_common.h"

namespace rt {
namespace paged {

typedef __attribute__((address_space(3))) void lds_void;
constexpr int PAGE = 64;

template <typename T> __device__ __forceinline__ float ld(const T* p);
template <> __device__ __forceinline__ float ld<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ld<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void st(T* p, float v);
template <> __device__ __forceinline__ void st<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void st<float>(float* p, float v) { *p = v; }

// v_exp_f32: arguments here are <= 0 (or -inf -> 0), where the library function's range handling does nothing
__device__ __forceinline__ float fexp2(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ bf16x8 pack_p(const f32x4& a, const f32x4& b) {
  uint4 v;
  v.x = pack2bf(a[0], a[1]);
  v.y = pack2bf(a[2], a[3]);
  v.z = pack2bf(b[0], b[1]);
  v.w = pack2bf(b[2], b[3]);
  return __builtin_bit_cast(bf16x8, v);
}
__device__ __forceinline__ bf16x8 cat4(const rt_s16x4& lo, const rt_s16x4& hi) {
  typedef __attribute__((ext_vector_type(8))) short s16x8;
  s16x8 v = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
  return __builtin_bit_cast(bf16x8, v);
}

struct Seg { int row, q_off, q_len, kv_off, kv_len, pos0, pad0, pad1; };  // 8 ints

// LDS image of a K (V) tile: rows of DQ (DV) elements, 16-B chunk c of row r at slot c ^ swizzle(r) (an
// involution, so the same function maps slots back to chunks). K: row reads conflict-free; V: transposed reads.
template <int DQ>
__device__ __forceinline__ int kq_chunk(int r, int c) {
  return c ^ ((DQ / 64) % 2 ? ((r >> 1) & 7) : (r & 15 & (DQ / 8 - 1)));
}
template <int DQ>
__device__ __forceinline__ int kq_off(int r, int c) {
  return r * (DQ * 2) + (kq_chunk<DQ>(r, c) << 4);
}
template <int DV>
__device__ __forceinline__ int vv_chunk(int r, int c) {
  constexpr int NCH = DV / 8, RPB = 128 / DV;
  return c ^ (((r / RPB) & (NCH / 2 - 1)) << 1);
}
template <int DV>
__device__ __forceinline__ int vv_off(int r, int c) {
  return r * (DV * 2) + (vv_chunk<DV>(r, c) << 4);
}

}  // namespace paged
}  // namespace rt
