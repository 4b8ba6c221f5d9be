// Mixture-of-experts feed-forward for gfx950: routing, the sort of (token, slot) pairs by expert, and
// the grouped expert products at few rows per expert (many rows per expert: the GRP form of
// gemm_big_kernel). All row counts stay on the device: every launch has a fixed grid, so a decode step
// with these kernels can be captured in a graph.
//
//   moe_route    logits [T, ldl] fp32, or nslab split-K slabs of them (columns [0, E) experts, optional column E = shared gate) ->
//                per token the `top` experts of the largest choice score softmax(z) + correction and
//                their weights softmax(z) (not renormalised), then `nshared` slots of the shared
//                expert (groups E .. E + nshared - 1) with weight sigmoid(shared gate);
//   moe_sort     one workgroup per group: stable counting sort of the pairs -> group offsets, the token
//                behind each sorted row, and the sorted row of each pair;
//   moe_tiles    256-row tiles of the sorted rows for the grouped token-parallel GEMM;
//   moe_rows     grouped product at few rows per group: weights streamed straight to registers as MFMA
//                operands (each read once per 64 rows), 4 waves splitting K, reduced through LDS;
//                PAIR: gate and up rows together with the gated linear unit in the epilogue.
#include "rt_common.h"

namespace rt {

// one wave per token
__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, long ldl, int nslab,
                                                        long sstride, const float* __restrict__ correction, int T, int E, int top,
                                                        int nshared, int gate_col, int* __restrict__ idx,
                                                        float* __restrict__ wt) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  constexpr int MAXV = 8;  // E <= 512
  const float* z = logits + (long)t * ldl;
  float s[MAXV], c[MAXV];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int e = lane + 64 * i;
    s[i] = -INFINITY;
    if (e < E) {
      s[i] = z[e];
      for (int q = 1; q < nslab; ++q) s[i] += z[q * sstride + e];
    }
    mx = fmaxf(mx, s[i]);
  }
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    s[i] = lane + 64 * i < E ? expf(s[i] - mx) : 0.f;
    sum += s[i];
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int e = lane + 64 * i;
    s[i] = s[i] / sum;
    c[i] = e < E ? s[i] + correction[e] : -INFINITY;
  }
  const int slots = top + nshared;
  // order-preserving integer keys: (score, lower expert first); 0 = taken or out of range. Every float,
  // also a NaN, has a place in this order, so a chosen expert is always a free one
  unsigned key[MAXV];
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const unsigned u = __float_as_uint(c[i]);
    key[i] = lane + 64 * i < E ? max(u & 0x80000000u ? ~u : u | 0x80000000u, 1u) : 0u;
  }
  for (int k = 0; k < top; ++k) {
    unsigned bk = 0, bi = 0;
#pragma unroll
    for (int i = 0; i < MAXV; ++i)
      if (64 * i < E && key[i] > bk) { bk = key[i]; bi = i; }
    unsigned long long best = ((unsigned long long)bk << 32) | (0xffffffffu - (lane + 64 * bi));
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const unsigned long long other = __shfl_xor(best, o, 64);
      best = other > best ? other : best;
    }
    const int e = (int)(0xffffffffu - (unsigned)best);
#pragma unroll
    for (int i = 0; i < MAXV; ++i)
      if (lane + 64 * i == e) {  // the owner lane records its choice
        key[i] = 0;
        idx[(long)t * slots + k] = e;
        wt[(long)t * slots + k] = s[i];
      }
  }
  if (lane < nshared) {
    idx[(long)t * slots + top + lane] = E + lane;
    float zg = 0.f;
    if (gate_col >= 0)
      for (int q = 0; q < nslab; ++q) zg += z[q * sstride + gate_col];
    wt[(long)t * slots + top + lane] = gate_col >= 0 ? 1.f / (1.f + expf(-zg)) : 1.f;
  }
}

// workgroup g: counts the pairs of lower groups (its offset), then places its own pairs in pair order.
// Four consecutive pairs per thread and pass.
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int* __restrict__ idx, int P, int slots, int G,
                                                        int* __restrict__ offs, int* __restrict__ row_tok,
                                                        int* __restrict__ pair_pos) {
  __shared__ int cnt[16][2];
  __shared__ int wsum[2][16];
  const int g = blockIdx.x, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  auto load4 = [&](int i0, int (&e)[4]) {
    if (i0 + 3 < P) {
      const int4 v = *(const int4*)(idx + i0);
      e[0] = v.x; e[1] = v.y; e[2] = v.z; e[3] = v.w;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) e[j] = i0 + j < P ? idx[i0 + j] : 0x7fffffff;
    }
  };
  int less = 0, mine = 0;
  for (int i0 = tid * 4; i0 < P; i0 += 4096) {
    int e[4];
    load4(i0, e);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      less += e[j] < g;
      mine += e[j] == g;
    }
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    less += __shfl_xor(less, o, 64);
    mine += __shfl_xor(mine, o, 64);
  }
  if (lane == 0) { cnt[w][0] = less; cnt[w][1] = mine; }
  __syncthreads();
  int base = 0, total = 0;
#pragma unroll
  for (int q = 0; q < 16; ++q) { base += cnt[q][0]; total += cnt[q][1]; }
  if (tid == 0) {
    offs[g] = base;
    if (g == G - 1) offs[G] = base + total;
  }
  if (total == 0) return;
  int run = base, ph = 0;
  for (int b0 = 0; b0 < P; b0 += 4096, ph ^= 1) {
    const int i0 = b0 + tid * 4;
    int e[4] = {-1, -1, -1, -1}, c = 0;
    if (i0 < P) load4(i0, e);
#pragma unroll
    for (int j = 0; j < 4; ++j) c += e[j] == g;
    int inc = c;  // inclusive scan over the wave
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int v = __shfl_up(inc, o, 64);
      if (lane >= o) inc += v;
    }
    if (lane == 63) wsum[ph][w] = inc;
    __syncthreads();
    int pos = run + inc - c, all = 0;
#pragma unroll
    for (int q = 0; q < 16; ++q) {
      const int v = wsum[ph][q];
      if (q < w) pos += v;
      all += v;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (e[j] == g) {
        row_tok[pos] = (i0 + j) / slots;
        pair_pos[i0 + j] = pos++;
      }
    run += all;
  }
}

__global__ __launch_bounds__(1024) void moe_tiles_kernel(const int* __restrict__ offs, int G, int rows, int max_tiles,
                                                         int4* __restrict__ tiles, int* __restrict__ n_tiles) {
  __shared__ int first[1025];
  const int g = threadIdx.x;
  if (g < G) first[g + 1] = (offs[g + 1] - offs[g] + rows - 1) / rows;
  if (g == 0) first[0] = 0;
  __syncthreads();
  if (g == 0)
    for (int i = 0; i < G; ++i) first[i + 1] += first[i];
  __syncthreads();
  if (g < G) {
    const int b = offs[g], e = offs[g + 1];
    for (int i = first[g]; i < first[g + 1] && i < max_tiles; ++i) {
      const int m0 = b + (i - first[g]) * rows;
      tiles[i] = make_int4(g, m0, min(m0 + rows, e), 0);
    }
  }
  if (g == 0) *n_tiles = min(first[G], max_tiles);
}

struct MoeRowsArgs {
  const bf16_t* A; long lda; const int* row_map;  // A row of sorted row r (null: r)
  const bf16_t* W; long sW, ldw;                  // group g: W + g * sW; PAIR: [gate; up], N rows each
  void* C; long ldc;
  const int* offs;
  int N, K;
  GluP glu;
};

// grid (N / 16, groups). Each wave takes K / 4 of the reduction in 32-deep MFMA steps, U steps of operands
// in registers and the next U in flight (non-temporal weight loads: with the compiler's own schedule this
// streamed 2.7 TB/s, with the explicit double buffer 4.6).
template <bool PAIR, bool OUT_F32, int MT>
__global__ __launch_bounds__(256) void moe_rows_kernel(MoeRowsArgs p) {
  constexpr int NB = PAIR ? 2 : 1;
  constexpr int U = MT == 4 ? 2 : 4;
  __shared__ float red[4][MT * NB][64 * 4];
  const int g = blockIdx.y, n0 = blockIdx.x * 16;
  const int beg = p.offs[g], end = p.offs[g + 1];
  if (beg >= end) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int r16 = lane & 15, q = lane >> 4;
  const bf16_t* W = p.W + (long)g * p.sW;
  const bf16_t* wp[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) wp[b] = W + (long)(b * p.N + min(n0 + r16, p.N - 1)) * p.ldw + 8 * q;
  const int steps = (p.K + 31) / 32;
  const int groups = (steps + U - 1) / U, per = (groups + 3) / 4;
  const int s0 = w * per, s1 = min(groups, s0 + per);
  for (int m0 = beg; m0 < end; m0 += 16 * MT) {
    const bf16_t* ap[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int r = min(m0 + 16 * i + r16, end - 1);
      ap[i] = p.A + (long)(p.row_map ? p.row_map[r] : r) * p.lda + 8 * q;
    }
    f32x4 acc[MT][NB];
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[i][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int mt = min(MT, (end - m0 + 15) / 16);
    bf16x8 wf[2][NB][U], af[2][MT][U];
    auto load = [&](int s, int d) {
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = (s * U + u) * 32;
        const bool ok = k + 8 * q < p.K;  // K % 8 == 0: a lane's 8 elements are all in or all out
#pragma unroll
        for (int b = 0; b < NB; ++b) wf[d][b][u] = ok ? __builtin_bit_cast(bf16x8, load_nt16(wp[b] + k)) : bf16x8{};
#pragma unroll
        for (int i = 0; i < MT; ++i) af[d][i][u] = ok ? *(const bf16x8*)(ap[i] + k) : bf16x8{};
      }
    };
    auto mul = [&](int d) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
          for (int b = 0; b < NB; ++b)
            acc[i][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af[d][i][u], wf[d][b][u], acc[i][b], 0, 0, 0);
    };
    if (s0 < s1) load(s0, 0);
    for (int s = s0; s < s1; s += 2) {
      if (s + 1 < s1) load(s + 1, 1);
      mul(0);
      if (s + 1 < s1) {
        if (s + 2 < s1) load(s + 2, 0);
        mul(1);
      }
    }
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int b = 0; b < NB; ++b) *(f32x4*)&red[w][i * NB + b][lane * 4] = acc[i][b];
    __syncthreads();
    // acc[r]: row 4 q + r, column r16; wave w finishes tiles w, w + 4, ...
    for (int i = w; i < mt; i += 4) {
      f32x4 v[NB];
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        v[b] = *(const f32x4*)&red[0][i * NB + b][lane * 4];
#pragma unroll
        for (int x = 1; x < 4; ++x) v[b] += *(const f32x4*)&red[x][i * NB + b][lane * 4];
      }
      const int col = n0 + r16;
      if (col < p.N) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = m0 + 16 * i + 4 * q + r;
          if (row >= end) continue;
          const float y = PAIR ? glu(v[0][r], v[NB - 1][r], p.glu) : v[0][r];
          if constexpr (OUT_F32) ((float*)p.C)[(long)row * p.ldc + col] = y;
          else ((bf16_t*)p.C)[(long)row * p.ldc + col] = f2bf(y);
        }
      }
    }
    __syncthreads();
  }
}

// Grouped product at up to 64 rows per group and pass, weights and rows through an LDS-DMA ring (the
// structure of gemm_m64_kernel): workgroup = 64 weight rows (PAIR: 32 gate + 32 up) of one group, 64-deep
// K-steps of X[64] and W[64] rows in a 4-slot ring, three steps in flight. Wave w owns rows [16 w, 16 w + 16)
// and skips their X loads and products when the group has none there. K % 64 == 0, N % 64 == 0 (PAIR: 32).
constexpr int RING_SLOTS = 4, RING_SLOT = 2 * 64 * 128;
__device__ __forceinline__ int ring_swz(int row) { return (row >> 1) & 7; }

template <bool PAIR, bool OUT_F32>
__global__ __launch_bounds__(256, 2) void moe_ring_kernel(MoeRowsArgs p) {
  typedef __attribute__((address_space(3))) void lds_void;
  __shared__ __attribute__((aligned(16))) char smem[RING_SLOTS * RING_SLOT];  // the only __shared__ object
  const int g = blockIdx.y, cg = blockIdx.x;
  const int beg = p.offs[g], end = p.offs[g + 1];
  if (beg >= end) return;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int frow = lane & 15, fq = lane >> 4;
  const int nk = p.K / 64;
  const bf16_t* W = p.W + (long)g * p.sW;
  const bf16_t* wp[2];
  int lr[2], ck[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    lr[j] = (wid * 2 + j) * 8 + (lane >> 3);
    ck[j] = ((lane & 7) ^ ring_swz(lr[j])) * 8;
    const int wr = PAIR ? (lr[j] < 32 ? cg * 32 + lr[j] : p.N + cg * 32 + lr[j] - 32) : cg * 64 + lr[j];
    wp[j] = W + (long)wr * p.ldw + ck[j];
  }
  for (int m0 = beg; m0 < end; m0 += 64) {
    const bool mine = m0 + 16 * wid < end;  // wave-uniform
    const bf16_t* xp[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int r = min(m0 + lr[j], end - 1);
      xp[j] = p.A + (long)(p.row_map ? p.row_map[r] : r) * p.lda + ck[j];
    }
    auto stage = [&](int t) {
      char* slot = smem + (t % RING_SLOTS) * RING_SLOT;
#pragma unroll
      for (int j = 0; j < 2; ++j)
        __builtin_amdgcn_global_load_lds((const void*)(wp[j] + t * 64), (lds_void*)(slot + 8192 + (wid * 2 + j) * 1024), 16, 0, 0);
      if (mine) {
#pragma unroll
        for (int j = 0; j < 2; ++j)
          __builtin_amdgcn_global_load_lds((const void*)(xp[j] + t * 64), (lds_void*)(slot + (wid * 2 + j) * 1024), 16, 0, 0);
      }
    };
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    // row pointers loaded above are in registers before the counted waits start
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
#pragma unroll
    for (int i = 0; i < RING_SLOTS - 1; ++i)
      if (i < nk) stage(i);
    for (int i = 0; i < nk; ++i) {
      const int ahead = min(RING_SLOTS - 2, nk - 1 - i);  // later steps stay in flight
      if (mine) {
        if (ahead >= 2) asm volatile("s_waitcnt vmcnt(8)" ::: "memory");
        else if (ahead == 1) asm volatile("s_waitcnt vmcnt(4)" ::: "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      } else {
        if (ahead >= 2) asm volatile("s_waitcnt vmcnt(4)" ::: "memory");
        else if (ahead == 1) asm volatile("s_waitcnt vmcnt(2)" ::: "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      }
      asm volatile("s_barrier" ::: "memory");
      // the slot read in the previous step is free: every wave is past it
      if (i + RING_SLOTS - 1 < nk) stage(i + RING_SLOTS - 1);
      if (!mine) continue;
      const char* slot = smem + (i % RING_SLOTS) * RING_SLOT;
      const int ar = wid * 16 + frow;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const int c = kk * 4 + fq;
        const bf16x8 a = *(const bf16x8*)(slot + ar * 128 + ((c ^ ring_swz(ar)) << 4));
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int br = j * 16 + frow;
          const bf16x8 b = *(const bf16x8*)(slot + 8192 + br * 128 + ((c ^ ring_swz(br)) << 4));
          acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[j], 0, 0, 0);
        }
      }
    }
    // lane holds C[16 wid + 4 fq + r][16 j + frow]
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = m0 + 16 * wid + 4 * fq + r;
      if (row >= end) continue;
#pragma unroll
      for (int j = 0; j < (PAIR ? 2 : 4); ++j) {
        const int col = (PAIR ? cg * 32 : cg * 64) + 16 * j + frow;
        const float y = PAIR ? glu(acc[j][r], acc[j + (PAIR ? 2 : 0)][r], p.glu) : acc[j][r];
        if constexpr (OUT_F32) ((float*)p.C)[(long)row * p.ldc + col] = y;
        else ((bf16_t*)p.C)[(long)row * p.ldc + col] = f2bf(y);
      }
    }
    // every wave has read its last slots before the next pass stages over them
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    asm volatile("s_barrier" ::: "memory");
  }
}

}  // namespace rt

using namespace rt;

extern "C" int rt_moe_route(const float* logits, long ldl, int nslab, long sstride, const float* correction, int T, int E, int top, int nshared,
                            int gate_col, int* idx, float* wt, hipStream_t stream) {
  if (T <= 0) return 0;
  if (E < 1 || E > 512 || top < 1 || top > E || nshared < 0 || nshared > 64) return -1;
  hipLaunchKernelGGL(moe_route_kernel, dim3((T + 3) / 4), dim3(256), 0, stream, logits, ldl, nslab, sstride, correction, T, E, top,
                     nshared, gate_col, idx, wt);
  RT_LAUNCH_CHECK();
  return 0;
}

// tiles / n_tiles may be null (few rows per group: no tile list)
extern "C" int rt_moe_sort(const int* idx, int P, int slots, int G, int* offs, int* row_tok, int* pair_pos,
                           int tile_rows, int max_tiles, void* tiles, int* n_tiles, hipStream_t stream) {
  if (P <= 0) return 0;
  if (G < 1 || G > 1024) return -1;
  hipLaunchKernelGGL(moe_sort_kernel, dim3(G), dim3(1024), 0, stream, idx, P, slots, G, offs, row_tok, pair_pos);
  if (tiles) {
    hipLaunchKernelGGL(moe_tiles_kernel, dim3(1), dim3(1024), 0, stream, offs, G, tile_rows, max_tiles, (int4*)tiles,
                       n_tiles);
  }
  RT_LAUNCH_CHECK();
  return 0;
}

// C[r] = A[row_map[r]] W_g^T (pair: gated linear unit of [gate; up] halves, N = half) for the rows of
// every group; mean_rows: expected rows per group (picks the row tiles per pass); ring: the LDS-DMA form
extern "C" int rt_moe_rows(const void* A, long lda, const int* row_map, const void* W, long sW, long ldw, void* C,
                           long ldc, const int* offs, int G, int N, int K, int pair, int out_f32, int mean_rows,
                           int ring, const float* glu_p, hipStream_t stream) {
  if (G <= 0 || N <= 0) return 0;
  if (K % 8 || ldw % 8 || lda % 8 || (pair && out_f32) || G > 65535) return -1;
  MoeRowsArgs p{(const bf16_t*)A, lda, row_map, (const bf16_t*)W, sW, ldw, C, ldc, offs, N, K, GluP{}};
  if (glu_p) { p.glu.limit = glu_p[0]; p.glu.alpha = glu_p[1]; p.glu.offset = glu_p[2]; }
  dim3 block(256);
  if (ring) {
    if (K % 64 || N % (pair ? 32 : 64)) return -3;
    dim3 rg(N / (pair ? 32 : 64), G);
    if (pair) hipLaunchKernelGGL((moe_ring_kernel<true, false>), rg, block, 0, stream, p);
    else if (out_f32) hipLaunchKernelGGL((moe_ring_kernel<false, true>), rg, block, 0, stream, p);
    else hipLaunchKernelGGL((moe_ring_kernel<false, false>), rg, block, 0, stream, p);
    RT_LAUNCH_CHECK();
    return 0;
  }
  dim3 grid((N + 15) / 16, G);
#define MR(MTV)                                                                                          \
  if (pair) hipLaunchKernelGGL((moe_rows_kernel<true, false, MTV>), grid, block, 0, stream, p);          \
  else if (out_f32) hipLaunchKernelGGL((moe_rows_kernel<false, true, MTV>), grid, block, 0, stream, p);  \
  else hipLaunchKernelGGL((moe_rows_kernel<false, false, MTV>), grid, block, 0, stream, p);
  if (mean_rows <= 12) { MR(1) }
  else if (mean_rows <= 28) { MR(2) }
  else { MR(4) }
#undef MR
  RT_LAUNCH_CHECK();
  return 0;
}
