// Grouped-query attention over a paged K/V cache with a sliding window and kept first tokens, for gfx950:
// query i sees key j <= i with i - j < size or j < keep; scores are (q . k) * scale, optionally softcapped
// (cap * tanh(s / cap)); query / key width D and value width V need not be equal.
//
// Cache: pool [pages][G heads][64 tokens][D + V] (a key row and its value row are one run; the keys of a head
// on a page are one contiguous block), page table [rows][max_pages] int32 (page 0 is never given to a
// request). Only the pages that hold kept or windowed keys are read, whatever the length of the context.
//
//   window_prep     q / k norm over the whole projection, rotation (halves), cache append
//   window_decode   few query tokens per request: (token, key head, partition of its visible tiles), then
//                   partition_merge
//   window_prefill  longer portions: flash attention straight from the pages (a 64-key tile is one page)
//   window_any      any size and fp32: one workgroup per (token, head)
#include "rt_paged.h"

#include <algorithm>

namespace rt {
namespace wa {

using namespace paged;

// ---------------------------------------------------------------------------------------------
// prep
// ---------------------------------------------------------------------------------------------
struct PrepArgs {
  void* proj; long ldp;        // [T, ldp]: q at q_col, k at k_col, v at v_col
  int q_col, k_col, v_col;
  const void* q_norm; const void* k_norm;             // [H * D], [G * D] (null: no norm)
  float eps;
  const float* cosT; const float* sinT; int max_pos;  // [max_pos, half]
  int half;                    // dimension i < half turns with i + half
  const int* row; const int* pos;
  void* pool; const int* tab; int max_pages, n_pages, n_rows;
  int H, G, D, V;
};

template <typename T, int N>
__device__ __forceinline__ void ldn(const T* p, float* o) {
  if constexpr (N == 8) unpack8(*(const uint4*)p, o);
  else o[0] = ld(p);
}
template <typename T, int N>
__device__ __forceinline__ void stn(T* p, const float* o) {
  if constexpr (N == 8) *(uint4*)p = pack8(o);
  else st(p, o[0]);
}

// N consecutive elements per access: 8 (bf16, D, V and half multiples of 8, aligned rows) or 1
template <typename T, int N>
__global__ __launch_bounds__(256) void window_prep_kernel(PrepArgs a) {
  __shared__ float sbuf[8];
  const int t = blockIdx.x, tid = threadIdx.x;
  T* pr = (T*)a.proj + (long)t * a.ldp;
  const int p_raw = a.pos[t], pos = min(max(p_raw, 0), a.max_pos - 1);
  const float* cs = a.cosT + (long)pos * a.half;
  const float* sn = a.sinT + (long)pos * a.half;
  const int row = a.row[t], pg = pos / PAGE;
  const bool ok = row >= 0 && row < a.n_rows && pg < a.max_pages;
  const int page = ok ? a.tab[(long)row * a.max_pages + pg] : -1;
  const bool append = page >= 0 && page < a.n_pages;
  T* dst = (T*)a.pool + ((long)max(page, 0) * a.G * PAGE + pos % PAGE) * (a.D + a.V);  // + head * PAGE * (D + V)
  const long hs = (long)PAGE * (a.D + a.V);

  auto squares = [&](const T* x, int n) {
    float s = 0.f, v[N];
    for (int e = tid * N; e < n; e += 256 * N) {
      ldn<T, N>(x + e, v);
#pragma unroll
      for (int k = 0; k < N; ++k) s += v[k] * v[k];
    }
    return s;
  };
  // one thread normalises and turns both halves of its pairs, so rows may be written in place
  auto turn = [&](T* x, const T* w, int heads, float rstd, bool to_cache) {
    for (int e = tid * N; e < heads * a.D; e += 256 * N) {
      const int h = e / a.D, i = e % a.D;
      if (i >= a.half && i < 2 * a.half) continue;
      T* o = to_cache ? dst + h * hs : x + h * a.D;
      float u[N], wu[N];
      ldn<T, N>(x + e, u);
      if (w) {
        ldn<T, N>(w + e, wu);
#pragma unroll
        for (int k = 0; k < N; ++k) u[k] *= rstd * wu[k];
      }
      if (i < a.half) {
        float v[N], r[N];
        ldn<T, N>(x + e + a.half, v);
        if (w) {
          ldn<T, N>(w + e + a.half, wu);
#pragma unroll
          for (int k = 0; k < N; ++k) v[k] *= rstd * wu[k];
        }
#pragma unroll
        for (int k = 0; k < N; ++k) {
          const float c = cs[i + k], s = sn[i + k];
          r[k] = v[k] * c + u[k] * s;
          u[k] = u[k] * c - v[k] * s;
        }
        if (!to_cache || append) stn<T, N>(o + i + a.half, r);
      }
      if (!to_cache || append) stn<T, N>(o + i, u);
    }
  };
  T* q = pr + a.q_col;
  T* k = pr + a.k_col;
  float rq = 1.f, rk = 1.f;
  if (a.q_norm || a.k_norm) {
    float sq = squares(q, a.H * a.D), sk = squares(k, a.G * a.D);
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((tid & 63) == 0) {
      sbuf[tid >> 6] = sq;
      sbuf[4 + (tid >> 6)] = sk;
    }
    __syncthreads();
    if (a.q_norm) rq = 1.f / sqrtf((sbuf[0] + sbuf[1] + sbuf[2] + sbuf[3]) / (a.H * a.D) + a.eps);
    if (a.k_norm) rk = 1.f / sqrtf((sbuf[4] + sbuf[5] + sbuf[6] + sbuf[7]) / (a.G * a.D) + a.eps);
  }
  turn(q, (const T*)a.q_norm, a.H, rq, false);
  turn(k, (const T*)a.k_norm, a.G, rk, true);
  if (append) {
    const T* v = pr + a.v_col;
    for (int e = tid * N; e < a.G * a.V; e += 256 * N) {
      T* o = dst + e / a.V * hs + a.D + e % a.V;
      if constexpr (N == 8) *(uint4*)o = *(const uint4*)(v + e);
      else *o = v[e];
    }
  }
}

// what a query at a position sees: [0, kept) and [lo, pos], and the tile lists that cover them
struct Mask {
  int size, keep;  // size: INT_MAX without a window
  __device__ __forceinline__ bool sees(int q, int k) const { return k <= q && (q - k < size || k < keep); }
  __device__ __forceinline__ int lo(int q) const { return q < size ? 0 : q - size + 1; }
};
template <int TILE>
struct Tiles {
  int kept, w0, n;  // tiles over kept keys before the window's first tile, that tile's key, all tiles
  // queries q0 .. q1
  __device__ __forceinline__ Tiles(const Mask& m, int q0, int q1) {
    w0 = m.lo(q0) / TILE * TILE;
    kept = (min(m.keep, w0) + TILE - 1) / TILE;
    n = kept + (q1 - w0) / TILE + 1;
  }
  __device__ __forceinline__ int key(int i) const { return i < kept ? i * TILE : w0 + (i - kept) * TILE; }
};

// score in log2 units: x = q . k
struct Score {
  float mul, cap2;  // without a cap: x * mul; with one: cap2 * tanh(x * scale / cap), mul = 2 log2(e) scale / cap
  __device__ __forceinline__ float operator()(float x) const {
    const float y = x * mul;
    return cap2 > 0.f ? cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(1.f + fexp2(y)) : y;
  }
};
static Score make_score(float scale, float cap) {
  const float l2e = 1.4426950408889634f;
  return cap > 0.f ? Score{2.f * l2e * scale / cap, cap * l2e} : Score{scale * l2e, 0.f};
}

// ---------------------------------------------------------------------------------------------
// decode: workgroup = (token, key head with its 16 NH query heads at most, partition), 4 waves
// ---------------------------------------------------------------------------------------------
// Per 32-key tile one LDS image [K: 64 QS columns | V: 64 RT columns], two buffers, LDS-DMA one tile ahead:
//   scores S^T = K Q^T (key on the MFMA row, head on the lane) by waves (key half, K-dim half) for NH = 1 and
//   (key half, head tile) for NH = 2, exchanged through LDS; every wave runs the same online softmax and
//   accumulates O^T += V^T P^T for its own quarter of the value columns (transposed reads of the image).
// A token's visible tiles are cut in NP equal partitions, so a captured launch with a fixed NP balances every
// length. Image rows are an odd number of 16-B chunks (row reads conflict-free).
struct DecArgs {
  const bf16_t* q; long ldq;  // [T, ldq], head h at h * D
  const bf16_t* pool; const int* tab; int max_pages, n_pages, n_rows;
  const int* row; const int* pos;
  float* part; float* ml;     // [T, H, NP, V], [T, H, NP, 2] (max in log2 units, sum)
  int H, G, D, V, NP;
  Mask mask;
  Score score;
};

template <int QS, int RT, int NH>
__global__ __launch_bounds__(256, 2) void window_decode_kernel(DecArgs a) {
  constexpr int CPR = 8 * QS + 8 * RT + 1, ROWB = CPR * 16;
  constexpr int NI = (32 * CPR + 255) / 256;         // LDS-DMA instructions per wave and tile
  constexpr int NIT = (32 * CPR + 63) / 64;          // of the workgroup (the last one may be half used)
  constexpr int BUFB = NIT * 1024;
  constexpr int QF = NH == 1 ? QS : 2 * QS;          // query fragments per wave
  __shared__ __attribute__((aligned(16))) char smem[2 * BUFB + 4096];
  float* sx = (float*)(smem + 2 * BUFB);             // [4 waves][64 lanes][4]
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g = lane >> 4, r16 = lane & 15;
  const int bid = xcd_remap(blockIdx.x, gridDim.x);
  const int part = bid % a.NP, gh = bid / a.NP % a.G, t = bid / (a.NP * a.G);
  const int HG = a.H / a.G, h0 = gh * HG;            // query heads h0 .. h0 + HG - 1
  const int row = min(max(a.row[t], 0), a.n_rows - 1);
  const int pos = min(max(a.pos[t], 0), a.max_pages * PAGE - 1);
  const Tiles<32> tl(a.mask, pos, pos);
  const int per = (tl.n + a.NP - 1) / a.NP;
  const int i0 = part * per, i1 = min(tl.n, i0 + per);
  if (i0 >= i1) {  // nothing for this partition (uniform over the workgroup)
    if (tid < HG) {
      float* m = a.ml + (((long)t * a.H + h0 + tid) * a.NP + part) * 2;
      m[0] = -INFINITY;
      m[1] = 0.f;
    }
    return;
  }
  // query fragments: lane holds Q[head r16][32 s + 8 g ..]; heads past the last repeat it (not stored)
  const int kt = w & 1, hi = w >> 1;                 // key half; K-dim half (NH = 1) or head tile (NH = 2)
  const int qh = h0 + min((NH == 2 ? hi * 16 : 0) + r16, HG - 1);
  const int sbase = NH == 1 ? hi * QS : 0;
  bf16x8 qf[QF];
  const bf16_t* qp = a.q + (long)t * a.ldq + (long)qh * a.D;
#pragma unroll
  for (int s = 0; s < QF; ++s) qf[s] = *(const bf16x8*)(qp + min(32 * (sbase + s) + 8 * g, a.D - 8));
  const int* tab = a.tab + (long)row * a.max_pages;
  const int W = a.D + a.V;

  // LDS-DMA sources: instruction j of wave w covers image chunks (4 j + w) * 64 + lane; columns past D (V)
  // repeat the last chunk (the query is zero there, the sums are not stored)
  uint32_t src[NI];  // element offset from the tile's first cache row
#pragma unroll
  for (int j = 0; j < NI; ++j) {
    const int c = (4 * j + w) * 64 + lane, cc = c % CPR;
    const int col = cc < 8 * QS ? min(8 * cc, a.D - 8) : a.D + min(8 * (cc - 8 * QS), a.V - 8);
    src[j] = (uint32_t)(min(c / CPR, 31) * W + col);
  }
  auto page_of = [&](int i) { return min(max(tab[tl.key(i) / PAGE], 0), a.n_pages - 1); };
  auto stage = [&](int i, int page, int buf) {
    const bf16_t* base = a.pool + (((long)page * a.G + gh) * PAGE + tl.key(i) % PAGE) * W;
#pragma unroll
    for (int j = 0; j < NI; ++j) {
      if (4 * j + w < NIT)  // wave-uniform
        __builtin_amdgcn_global_load_lds((const void*)(base + src[j]), (lds_void*)(smem + buf * BUFB + (4 * j + w) * 1024),
                                         16, 0, 0);
    }
  };

  f32x4 o[NH][RT];
#pragma unroll
  for (int n = 0; n < NH; ++n)
#pragma unroll
    for (int c = 0; c < RT; ++c) o[n][c] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m[NH], l[NH];
#pragma unroll
  for (int n = 0; n < NH; ++n) { m[n] = -INFINITY; l[n] = 0.f; }

  const bool more = w < NIT % 4;  // this wave issues NIT / 4 + 1 instructions per tile, else NIT / 4
  stage(i0, page_of(i0), 0);
  if (i0 + 1 < i1) stage(i0 + 1, page_of(i0 + 1), 1);
  if (a.D < 64 * QS) {
#pragma unroll
    for (int s = 0; s < QF; ++s)
      if (32 * (sbase + s) + 8 * g >= a.D) qf[s] = bf16x8{};
  }
#pragma unroll
  for (int s = 0; s < QF; ++s) asm volatile("" : "+v"(qf[s]));
  int buf = 0;
  for (int i = i0; i < i1; ++i, buf ^= 1) {
    const bool n1 = i + 1 < i1, n2 = i + 2 < i1;
    const int page2 = n2 ? page_of(i + 2) : 0;
    const int key0 = tl.key(i);
    // this tile's image; the next tile's instructions stay in flight
    if (!n1) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    else if (more) asm volatile("s_waitcnt vmcnt(%0)" :: "n"(NIT / 4 + 1) : "memory");
    else asm volatile("s_waitcnt vmcnt(%0)" :: "n"(NIT / 4) : "memory");
    asm volatile("s_barrier" ::: "memory");           // ... of every wave
    const char* img = smem + buf * BUFB;
    // ---- scores ----
    f32x4 sp[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};  // two independent MFMA chains
    {
      const char* kp = img + (16 * kt + r16) * ROWB + (4 * sbase + g) * 16;
#pragma unroll
      for (int s = 0; s < QF; ++s) {
        const bf16x8 kf = *(const bf16x8*)(kp + s * 64);
        sp[s & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s], sp[s & 1], 0, 0, 0);
      }
    }
    *(f32x4*)(sx + (w * 64 + lane) * 4) = sp[0] + sp[1];
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    asm volatile("s_barrier" ::: "memory");
    // ---- softmax (identical in every wave) ----
    const bool whole = key0 + 31 <= pos && (pos - key0 < a.mask.size || key0 + 31 < a.mask.keep);
    bf16x8 pa[NH];
#pragma unroll
    for (int n = 0; n < NH; ++n) {
      f32x4 s2[2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        if constexpr (NH == 1)
          s2[k] = *(const f32x4*)(sx + (k * 64 + lane) * 4) + *(const f32x4*)(sx + ((k + 2) * 64 + lane) * 4);
        else
          s2[k] = *(const f32x4*)(sx + ((k + 2 * n) * 64 + lane) * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) s2[k][e] = a.score(s2[k][e]);
      }
      if (!whole) {
#pragma unroll
        for (int k = 0; k < 2; ++k)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (!a.mask.sees(pos, key0 + 16 * k + 4 * g + e)) s2[k][e] = -INFINITY;
      }
      float mx = fmaxf(fmaxf(fmaxf(s2[0][0], s2[0][1]), fmaxf(s2[0][2], s2[0][3])),
                       fmaxf(fmaxf(s2[1][0], s2[1][1]), fmaxf(s2[1][2], s2[1][3])));
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[n], mx);  // finite: every listed tile holds a visible key
      const float alpha = fexp2(m[n] - mn);
      m[n] = mn;
      float rs = 0.f;
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float p = fexp2(s2[k][e] - mn);
          s2[k][e] = p;
          rs += p;
        }
      rs += __shfl_xor(rs, 16, 64);
      rs += __shfl_xor(rs, 32, 64);
      l[n] = l[n] * alpha + rs;
      pa[n] = pack_p(s2[0], s2[1]);
      // O^T: the head is the lane's column, as in the scores (most tiles bring no new maximum)
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int c = 0; c < RT; ++c) o[n][c] *= alpha;
      }
    }
    // ---- O += P V: value columns [16 RT w, 16 RT (w + 1)) ----
    const uint32_t va = lds_addr(img + (4 * g + ((lane >> 2) & 3)) * ROWB + 128 * QS + w * RT * 32 + (lane & 3) * 8);
    rt_s16x4 v[2 * RT];
    if constexpr (RT == 4) ds_tr16_frag2<16 * ROWB, 32, 32 + 16 * ROWB>(va, va + 64, v);
    else ds_tr16_x4<16 * ROWB, 32, 32 + 16 * ROWB>(va, v[0], v[1], v[2], v[3]);
#pragma unroll
    for (int c = 0; c < RT; ++c) {
      const bf16x8 vf = cat4(v[2 * c], v[2 * c + 1]);
#pragma unroll
      for (int n = 0; n < NH; ++n) o[n][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pa[n], o[n][c], 0, 0, 0);
    }
    if (n2) {  // every wave is done with this image: the tile after the next one takes its place
      asm volatile("s_barrier" ::: "memory");
      stage(i + 2, page2, buf);
    }
  }
  // o[n][c][e]: head h0 + 16 n + r16, value column 16 (RT w + c) + 4 g + e
#pragma unroll
  for (int n = 0; n < NH; ++n) {
    if (16 * n + r16 >= HG) continue;
    const long th = ((long)t * a.H + h0 + 16 * n + r16) * a.NP + part;
    float* po = a.part + th * a.V + 16 * RT * w + 4 * g;
#pragma unroll
    for (int c = 0; c < RT; ++c)
      if (16 * (RT * w + c) + 4 * g < a.V) *(f32x4*)(po + 16 * c) = o[n][c];  // V % 8 == 0
    if (w == 0 && g == 0) *(float2*)(a.ml + th * 2) = make_float2(m[n], l[n]);
  }
}

// ---------------------------------------------------------------------------------------------
// prefill: 128 query rows of one head per workgroup, 4 waves x 32 rows, 64-key tiles = pages
// ---------------------------------------------------------------------------------------------
// Swapped S^T = K Q^T, P straight into the next MFMA (O^T = V^T P^T), double-buffered K / V tiles by LDS-DMA
// straight from the pages, one barrier per tile.
struct PreArgs {
  const bf16_t* q; long ldq;     // [tokens, ldq], head h at h * D, normed and rotated
  const bf16_t* pool; const int* tab; int max_pages, n_pages, n_rows;
  bf16_t* o; long ldo;
  const Seg* segs; const int2* tiles; int n_tiles;   // {segment, first query row / 128}
  int H, G, D, V;
  Mask mask;
  Score score;
  float out_scale;
};

template <int DQ, int DV>
__global__ __launch_bounds__(256, 2) void window_prefill_kernel(PreArgs a) {
  constexpr int NQ = DQ / 8, NV = DV / 8, DS = DQ / 32, DT = DV / 16;
  constexpr int KB = 64 * DQ * 2, VB = 64 * DV * 2;
  constexpr int OROW = DV + 8;
  constexpr int TILES = 2 * (KB + VB), OB = 128 * OROW * 2;
  __shared__ __attribute__((aligned(16))) char smem[TILES > OB ? TILES : OB];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g = lane >> 4, r16 = lane & 15;
  const int lin = xcd_remap(blockIdx.x, gridDim.x);
  const int h = lin / a.n_tiles, gh = h / (a.H / a.G);
  const int2 tile = a.tiles[lin % a.n_tiles];
  const Seg sg = a.segs[tile.x];
  const int qblk0 = tile.y * 128, q0 = qblk0 + wid * 32;
  const int pa0 = sg.pos0 + qblk0, pa1 = sg.pos0 + min(qblk0 + 128, sg.q_len) - 1;  // positions of the workgroup
  const Tiles<64> tl(a.mask, pa0, pa1);
  const int* tab = a.tab + (long)min(max(sg.row, 0), a.n_rows - 1) * a.max_pages;
  const int W = a.D + a.V;

  bf16x8 qf[2][DS];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int qr = min(q0 + 16 * u + r16, sg.q_len - 1);
    const bf16_t* qp = a.q + (long)(sg.q_off + qr) * a.ldq + (long)h * a.D;
#pragma unroll
    for (int s = 0; s < DS; ++s) {
      const int c = 32 * s + 8 * g;
      qf[u][s] = c < a.D ? *(const bf16x8*)(qp + c) : bf16x8{};
    }
  }
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int s = 0; s < DS; ++s) asm volatile("" : "+v"(qf[u][s]));

  f32x4 o[2][DT];
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int c = 0; c < DT; ++c) o[u][c] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m[2], l[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) { m[u] = -INFINITY; l[u] = 0.f; }

  // LDS-DMA of one tile: instruction j of this wave fills 1 KiB of the K (V) image; the lane's source chunk
  // undoes the image's swizzle. Columns past D (V) repeat the first chunk (the query is zero there, the
  // values are not stored); slots of the page past the request's keys are finite and masked.
  constexpr int JK = KB / 4096, JV = VB / 4096;
  uint32_t off[JK + JV];
#pragma unroll
  for (int j = 0; j < JK + JV; ++j) {
    const bool v = j >= JK;
    const int e = (4 * (v ? j - JK : j) + wid) * 64 + lane;
    const int key = v ? e / NV : e / NQ;
    const int c = 8 * (v ? vv_chunk<DV>(key, e % NV) : kq_chunk<DQ>(key, e % NQ));
    off[j] = (uint32_t)(key * W + (v ? a.D + (c < a.V ? c : 0) : (c < a.D ? c : 0)));
  }
  auto page_of = [&](int i) {
    const int p = tl.key(min(i, tl.n - 1)) / PAGE;
    return min(max(tab[min(p, a.max_pages - 1)], 0), a.n_pages - 1);
  };
  auto stage = [&](int page, int buf) {
    char* kd = smem + buf * (KB + VB);
    const bf16_t* base = a.pool + ((long)page * a.G + gh) * PAGE * W;
#pragma unroll
    for (int j = 0; j < JK + JV; ++j)
      __builtin_amdgcn_global_load_lds((const void*)(base + off[j]),
                                       (lds_void*)(kd + (j < JK ? 4 * j : KB / 1024 + 4 * (j - JK)) * 1024 + wid * 1024), 16, 0, 0);
  };
  stage(page_of(0), 0);
  int page = page_of(1);
  int cur = 0;
  for (int i = 0; i < tl.n; ++i, cur ^= 1) {
    const int kv0 = tl.key(i);
    const int page_next = page_of(i + 2);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this tile (issued one tile ago)
    asm volatile("s_barrier" ::: "memory");           // ... of every wave; the other buffer is free
    if (i + 1 < tl.n) stage(page, cur ^ 1);
    page = page_next;
    char* Ks = smem + cur * (KB + VB);
    char* Vs = Ks + KB;
    f32x4 stt[4][2];
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int u = 0; u < 2; ++u) stt[t][u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int s = 0; s < DS; ++s) {
        const bf16x8 kf = *(const bf16x8*)(Ks + kq_off<DQ>(16 * t + r16, 4 * s + g));
#pragma unroll
        for (int u = 0; u < 2; ++u)
          stt[t][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[u][s], stt[t][u], 0, 0, 0);
      }
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int e = 0; e < 4; ++e) stt[t][u][e] = a.score(stt[t][u][e]);
    const int w0 = sg.pos0 + q0, w1 = w0 + 31;  // positions of the wave's rows
    if (!(kv0 + 63 <= w0 && (w1 - kv0 < a.mask.size || kv0 + 63 < a.mask.keep))) {  // not all visible
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (!a.mask.sees(w0 + 16 * u + r16, kv0 + 16 * t + 4 * g + e)) stt[t][u][e] = -INFINITY;
    }
    float alpha[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float mx = -INFINITY;
#pragma unroll
      for (int t = 0; t < 4; ++t)
        mx = fmaxf(mx, fmaxf(fmaxf(stt[t][u][0], stt[t][u][1]), fmaxf(stt[t][u][2], stt[t][u][3])));
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[u], mx);
      const float mz = mn == -INFINITY ? 0.f : mn;  // a row may see nothing of its first tiles
      alpha[u] = fexp2(m[u] - mz);
      m[u] = mn;
      float rs = 0.f;
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float p = fexp2(stt[t][u][e] - mz);
          stt[t][u][e] = p;
          rs += p;
        }
      rs += __shfl_xor(rs, 16, 64);
      rs += __shfl_xor(rs, 32, 64);
      l[u] = l[u] * alpha[u] + rs;
    }
    // O^T: the query is the lane's column, as in the scores (most tiles bring no new maximum)
    if (__any(alpha[0] != 1.f || alpha[1] != 1.f)) {
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int c = 0; c < DT; ++c) o[u][c] *= alpha[u];
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 pa[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) pa[u] = pack_p(stt[2 * ks][u], stt[2 * ks + 1][u]);
      const int qrow = lane >> 2 & 3, pcol = lane & 3;
      const int key_a = 32 * ks + 4 * g + qrow;
#pragma unroll
      for (int c = 0; c < DT; c += 2) {
        const uint32_t a0 = lds_addr(Vs + vv_off<DV>(key_a, 2 * c + (pcol >> 1)) + ((pcol & 1) << 3));
        const uint32_t a1 = lds_addr(Vs + vv_off<DV>(key_a, 2 * c + 2 + (pcol >> 1)) + ((pcol & 1) << 3));
        rt_s16x4 l0, h0, l1, h1;
        ds_tr16_2x2<16 * DV * 2>(a0, a1, l0, h0, l1, h1);
        const bf16x8 v0 = cat4(l0, h0), v1 = cat4(l1, h1);
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          o[u][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v0, pa[u], o[u][c], 0, 0, 0);
          o[u][c + 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v1, pa[u], o[u][c + 1], 0, 0, 0);
        }
      }
    }
  }
  __syncthreads();  // the last tile's images become the O staging area
  bf16_t* Os = (bf16_t*)smem;
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const float sc = a.out_scale / l[u];  // a position sees itself
    const int r = wid * 32 + 16 * u + r16;
#pragma unroll
    for (int c = 0; c < DT; ++c)
      *(uint2*)(Os + r * OROW + 16 * c + 4 * g) =
          make_uint2(pack2bf(o[u][c][0] * sc, o[u][c][1] * sc), pack2bf(o[u][c][2] * sc, o[u][c][3] * sc));
  }
  __syncthreads();
  for (int e = tid; e < 128 * NV; e += 256) {
    const int r = e / NV, c = (e % NV) * 8;
    if (qblk0 + r < sg.q_len && c < a.V)
      *(uint4*)(a.o + (long)(sg.q_off + qblk0 + r) * a.ldo + (long)h * a.V + c) = *(const uint4*)(Os + r * OROW + c);
  }
}

// ---------------------------------------------------------------------------------------------
// any size and type: one workgroup per (head, token), 256 of its visible keys at a time
// ---------------------------------------------------------------------------------------------
struct AnyArgs {
  const void* q; long ldq;
  const void* pool; const int* tab; int max_pages, n_pages, n_rows;
  const int* row; const int* pos;
  void* o; long ldo;
  int H, G, D, V;
  Mask mask;
  float scale, cap, out_scale;
};

template <typename T>
__global__ __launch_bounds__(256) void window_any_kernel(AnyArgs a) {
  extern __shared__ float sm[];  // q [D], acc [V], p [256], key row offsets [256], sbuf [4]
  float* qs = sm;
  float* acc = qs + a.D;
  float* ps = acc + a.V;
  int* ks = (int*)(ps + 256);
  float* sbuf = (float*)(ks + 256);
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, gh = h / (a.H / a.G), W = a.D + a.V;
  const int row = min(max(a.row[t], 0), a.n_rows - 1);
  const int pos = min(max(a.pos[t], 0), a.max_pages * PAGE - 1);
  const int lo = a.mask.lo(pos), kept = min(a.mask.keep, lo), n = kept + pos - lo + 1;
  const int* tab = a.tab + (long)row * a.max_pages;
  for (int c = tid; c < a.D; c += 256) qs[c] = ld((const T*)a.q + (long)t * a.ldq + (long)h * a.D + c);
  for (int c = tid; c < a.V; c += 256) acc[c] = 0.f;
  float m = -INFINITY, l = 0.f;
  __syncthreads();
  for (int j0 = 0; j0 < n; j0 += 256) {
    const int j = j0 + tid;
    float s = -INFINITY;
    if (j < n) {
      const int key = j < kept ? j : lo + j - kept;
      const int page = min(max(tab[key / PAGE], 0), a.n_pages - 1);
      const int at = (page * a.G + gh) * PAGE + key % PAGE;  // pages * G * 64 fits an int (launcher)
      ks[tid] = at;
      const T* kp = (const T*)a.pool + (long)at * W;
      float d = 0.f;
      for (int c = 0; c < a.D; ++c) d = fmaf(qs[c], ld(kp + c), d);
      s = d * a.scale;
      if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
    }
    const float mn = fmaxf(m, block_max(s, sbuf));
    const float alpha = expf(m - mn);
    const float p = j < n ? expf(s - mn) : 0.f;
    ps[tid] = p;
    l = l * alpha + block_sum(p, sbuf);
    m = mn;
    __syncthreads();
    const int cnt = min(256, n - j0);
    for (int c = tid; c < a.V; c += 256) {
      float y = acc[c] * alpha;
      for (int k = 0; k < cnt; ++k) y = fmaf(ps[k], ld((const T*)a.pool + (long)ks[k] * W + a.D + c), y);
      acc[c] = y;
    }
    __syncthreads();
  }
  for (int c = tid; c < a.V; c += 256) st((T*)a.o + (long)t * a.ldo + (long)h * a.V + c, acc[c] / l * a.out_scale);
}

static Mask make_mask(int size, int keep) { return Mask{size > 0 ? size : 0x7fffffff, std::max(keep, 0)}; }

}  // namespace wa
}  // namespace rt

using namespace rt;
using namespace rt::wa;

extern "C" int rt_window_prep(int f32, void* proj, long ldp, int q_col, int k_col, int v_col, const void* q_norm,
                              const void* k_norm, float eps, const float* cosT, const float* sinT, int max_pos, int half,
                              const int* row, const int* pos, void* pool, const int* tab, int max_pages, int n_pages,
                              int n_rows, int T, int H, int G, int D, int V, hipStream_t stream) {
  if (T <= 0) return 0;
  if (2 * half > D || max_pos < 1) return -1;
  PrepArgs a{proj, ldp, q_col, k_col, v_col, q_norm, k_norm, eps, cosT, sinT, max_pos, half, row, pos,
             pool, tab, max_pages, n_pages, n_rows, H, G, D, V};
  const bool vec = !f32 && D % 8 == 0 && V % 8 == 0 && half % 8 == 0 && ldp % 8 == 0 && q_col % 8 == 0 && k_col % 8 == 0 &&
                   v_col % 8 == 0 && ((uintptr_t)proj | (uintptr_t)pool | (uintptr_t)q_norm | (uintptr_t)k_norm) % 16 == 0;
  if (f32) hipLaunchKernelGGL((window_prep_kernel<float, 1>), dim3(T), dim3(256), 0, stream, a);
  else if (vec) hipLaunchKernelGGL((window_prep_kernel<bf16_t, 8>), dim3(T), dim3(256), 0, stream, a);
  else hipLaunchKernelGGL((window_prep_kernel<bf16_t, 1>), dim3(T), dim3(256), 0, stream, a);
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_window_decode_ok(int H, int G, int D, int V) {
  return G > 0 && H % G == 0 && H / G <= 32 && D % 8 == 0 && V % 8 == 0 && D >= 8 && V >= 8 && D <= 256 && V <= 256;
}

extern "C" int rt_window_decode(const void* q, long ldq, const void* pool, const int* tab, int max_pages, int n_pages,
                                int n_rows, const int* row, const int* pos, float* part, float* ml, int T, int H, int G,
                                int D, int V, int NP, int size, int keep, float scale, float cap, hipStream_t stream) {
  if (T <= 0) return 0;
  if (!rt_window_decode_ok(H, G, D, V) || NP < 1 || ldq % 8) return -1;
  DecArgs a{(const bf16_t*)q, ldq, (const bf16_t*)pool, tab, max_pages, n_pages, n_rows, row, pos, part, ml, H, G, D, V, NP,
            make_mask(size, keep), make_score(scale, cap)};
  dim3 grid((unsigned)((long)T * G * NP)), block(256);
#define WD_(QS, RT)                                                                                        \
  do {                                                                                                     \
    if (H / G <= 16) hipLaunchKernelGGL((window_decode_kernel<QS, RT, 1>), grid, block, 0, stream, a);     \
    else hipLaunchKernelGGL((window_decode_kernel<QS, RT, 2>), grid, block, 0, stream, a);                 \
  } while (0)
#define WD_V(QS) do { if (V <= 128) WD_(QS, 2); else WD_(QS, 4); } while (0)
  if (D <= 64) WD_V(1);
  else if (D <= 128) WD_V(2);
  else if (D <= 192) WD_V(3);
  else WD_V(4);
#undef WD_V
#undef WD_
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_window_prefill_ok(int D, int V) { return D % 8 == 0 && V % 8 == 0 && D >= 8 && V >= 8 && D <= 256 && V <= 128; }

extern "C" int rt_window_prefill(const void* q, long ldq, const void* pool, const int* tab, int max_pages, int n_pages,
                                 int n_rows, void* o, long ldo, const void* segs, const void* tiles, int n_tiles, int H,
                                 int G, int D, int V, int size, int keep, float scale, float cap, float out_scale,
                                 hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (!rt_window_prefill_ok(D, V) || G < 1 || H % G || ldq % 8 || ldo % 8 || (uintptr_t)o % 16) return -1;
  PreArgs a{(const bf16_t*)q, ldq, (const bf16_t*)pool, tab, max_pages, n_pages, n_rows, (bf16_t*)o, ldo, (const Seg*)segs,
            (const int2*)tiles, n_tiles, H, G, D, V, make_mask(size, keep), make_score(scale, cap), out_scale};
  dim3 grid((unsigned)((long)n_tiles * H)), block(256);
#define WP_(DQ)                                                                                      \
  do {                                                                                               \
    if (V <= 64) hipLaunchKernelGGL((window_prefill_kernel<DQ, 64>), grid, block, 0, stream, a);     \
    else hipLaunchKernelGGL((window_prefill_kernel<DQ, 128>), grid, block, 0, stream, a);            \
  } while (0)
  if (D <= 64) WP_(64);
  else if (D <= 128) WP_(128);
  else if (D <= 192) WP_(192);
  else WP_(256);
#undef WP_
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_window_any(int f32, const void* q, long ldq, const void* pool, const int* tab, int max_pages, int n_pages,
                             int n_rows, const int* row, const int* pos, void* o, long ldo, int T, int H, int G, int D,
                             int V, int size, int keep, float scale, float cap, float out_scale, hipStream_t stream) {
  if (T <= 0) return 0;
  if (G < 1 || H % G || (long)n_pages * G * PAGE > 0x7fffffffL) return -1;
  const size_t lds = (size_t)(D + V + 512 + 4) * 4;
  if (lds > 65536) return -2;
  for (int t0 = 0; t0 < T; t0 += 65535) {
    const size_t es = f32 ? 4 : 2;
    AnyArgs a{(const char*)q + (long)t0 * ldq * es, ldq, pool, tab, max_pages, n_pages, n_rows, row + t0, pos + t0,
              (char*)o + (long)t0 * ldo * es, ldo, H, G, D, V, make_mask(size, keep), scale, cap, out_scale};
    dim3 grid(H, std::min(T - t0, 65535));
    if (f32) hipLaunchKernelGGL((window_any_kernel<float>), grid, dim3(256), lds, stream, a);
    else hipLaunchKernelGGL((window_any_kernel<bf16_t>), grid, dim3(256), lds, stream, a);
    RT_LAUNCH_CHECK();
  }
  return 0;
}
