// Latent attention for gfx950: per token one normed latent c [rank] and one rotated key part kr [rot]
// shared by all heads are cached (a row of KD = rank + rot in a paged pool); per head
//   k = [W_uk c, kr],  v = W_uv c,  score = (q_unrotated . W_uk c + q_rotated . kr) * scale,
// softmax whose denominator also holds exp(sink_h), output times sigmoid(gate).
//
// Cache: pool [pages][64][KD], page table [rows][max_pages] int32 (page 0 is never given to a request:
// rows without one point at it). A token of the batch is (row, position); its keys are 0 .. position.
//
// Few query tokens per request (decode, short portions) run the absorbed form: the query is moved into
// latent space once (q_abs = [W_uk^T q_unrotated, q_rotated], KD wide), so scores and the weighted sum
// both read the cached rows directly and all heads share them:
//   latent_prep -> head product (absorb) -> latent_decode (split over key partitions) -> latent_merge ->
//   head product (value expansion, gate)
// Longer portions expand the request's keys and values once per layer (a GEMM over the gathered rows)
// and run a flash kernel over [unrotated | rotated] heads:
//   latent_prep -> latent_gather -> (expand GEMM) -> latent_prefill
// latent_any is the absorbed attention for any size and for fp32 (one workgroup per token and head).
#include "rt_paged.h"

#include <algorithm>

namespace rt {
namespace la {

using namespace paged;

// ---------------------------------------------------------------------------------------------
// prep: latent norm + rotation + cache append (layers with a latent of their own), query rotation
// ---------------------------------------------------------------------------------------------
struct PrepArgs {
  void* proj; long ldp;        // [T, ldp]: q at 0 (heads of dim + rot), dkv at kv_col (rank + rot)
  int kv_col;                  // < 0: the layer reads another layer's cache
  const void* norm_w; float eps;
  const float* cosT; const float* sinT; int max_pos;  // [max_pos, rdims / 2], multiplier included
  int rdims;                   // rotated leading dimensions of the rot part (interleaved pairs)
  const int* row; const int* pos;
  void* pool; const int* tab; int max_pages, n_pages, n_rows;
  void* qabs; int n_abs;       // tokens [0, n_abs): rotated query part to qabs [.., H, rank + rot]; others in place
  int H, dim, rot, rank;
  int vec;                     // 16-B aligned rows and whole rotation: vector loads of the query part
};

template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(PrepArgs a) {
  __shared__ float sbuf[4];
  const int t = blockIdx.x, tid = threadIdx.x;
  T* pr = (T*)a.proj + (long)t * a.ldp;
  const int pos = min(max(a.pos[t], 0), a.max_pos - 1);
  const int half = a.rdims / 2, KD = a.rank + a.rot;
  const float* cs = a.cosT + (long)pos * half;
  const float* sn = a.sinT + (long)pos * half;
  if (a.kv_col >= 0) {
    const int row = a.row[t];
    const int pg_i = pos / PAGE;
    const bool ok = row >= 0 && row < a.n_rows && pg_i < a.max_pages;
    const int page = ok ? a.tab[(long)row * a.max_pages + pg_i] : -1;
    T* src = pr + a.kv_col;
    float s = 0.f;
    for (int c = tid; c < a.rank; c += 256) {
      const float v = ld(src + c);
      s += v * v;
    }
    const float rstd = 1.f / sqrtf(block_sum(s, sbuf) / a.rank + a.eps);
    if (page >= 0 && page < a.n_pages) {
      T* dst = (T*)a.pool + ((long)page * PAGE + pos % PAGE) * KD;
      for (int c = tid; c < a.rank; c += 256) st(dst + c, ld(src + c) * rstd * ld((const T*)a.norm_w + c));
      for (int i = tid; i < a.rot / 2; i += 256) {
        const float u = ld(src + a.rank + 2 * i), v = ld(src + a.rank + 2 * i + 1);
        const bool r = i < half;
        st(dst + a.rank + 2 * i, r ? u * cs[i] - v * sn[i] : u);
        st(dst + a.rank + 2 * i + 1, r ? v * cs[i] + u * sn[i] : v);
      }
    }
  }
  const int hp = a.rot / 2;
  if (sizeof(T) == 2 && a.vec) {  // 4 pairs = 16 B at a time
    const int h4 = hp / 4;
    for (int e = tid; e < a.H * h4; e += 256) {
      const int h = e / h4, i = (e % h4) * 4;
      T* q = pr + (long)h * (a.dim + a.rot) + a.dim + 2 * i;
      float x[8], y[8];
      unpack8(*(const uint4*)q, x);
      const float4 c = *(const float4*)(cs + i), s = *(const float4*)(sn + i);
      const float c4[4] = {c.x, c.y, c.z, c.w}, s4[4] = {s.x, s.y, s.z, s.w};
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        y[2 * k] = x[2 * k] * c4[k] - x[2 * k + 1] * s4[k];
        y[2 * k + 1] = x[2 * k + 1] * c4[k] + x[2 * k] * s4[k];
      }
      T* d = t < a.n_abs ? (T*)a.qabs + ((long)t * a.H + h) * KD + a.rank + 2 * i : q;
      *(uint4*)d = pack8(y);
    }
    return;
  }
  for (int e = tid; e < a.H * hp; e += 256) {
    const int h = e / hp, i = e % hp;
    T* q = pr + (long)h * (a.dim + a.rot) + a.dim + 2 * i;
    const float u = ld(q), v = ld(q + 1);
    const bool r = i < half;
    T* d = t < a.n_abs ? (T*)a.qabs + ((long)t * a.H + h) * KD + a.rank + 2 * i : q;
    st(d, r ? u * cs[i] - v * sn[i] : u);
    st(d + 1, r ? v * cs[i] + u * sn[i] : v);
  }
}

// ---------------------------------------------------------------------------------------------
// per-head product at few rows: C[t][b][:] = A[t][b][:] W_b^T (absorb: rank x dim per head; value
// expansion: vdim x rank, times sigmoid(gate[t][b N + n])). MFMA, weights streamed straight to registers. grid (N / 64, batch, T / (16 MT)), wave = 16 columns x 16 MT rows.
// ---------------------------------------------------------------------------------------------
template <int MT>
__global__ __launch_bounds__(256) void head_gemm_kernel(const bf16_t* __restrict__ A, long lda, long sA,
                                                        const bf16_t* __restrict__ W, long ldw, long sW,
                                                        bf16_t* __restrict__ C, long ldc, long sC, int T, int N, int K,
                                                        const bf16_t* __restrict__ gate, long ldg, int vec) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, q = lane >> 4;
  const int n0 = blockIdx.x * 64 + w * 16, b = blockIdx.y, t0 = blockIdx.z * 16 * MT;
  __shared__ __attribute__((aligned(16))) bf16_t tile[16 * MT][72];  // 64 columns, padded rows
  const bf16_t* ap[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) ap[i] = A + (long)min(t0 + 16 * i + r16, T - 1) * lda + b * sA + 8 * q;
  const bf16_t* wp = W + b * sW + (long)min(n0 + r16, N - 1) * ldw + 8 * q;
  // weight as the A operand: acc[i][r] = C[t0 + 16 i + r16][n0 + 4 q + r]
  f32x4 acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int U = MT == 1 ? 8 : 4;  // steps' operands in flight
  int k = 0;
  for (; k + 32 * U <= K; k += 32 * U) {
    bf16x8 wf[U], af[MT][U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      wf[u] = *(const bf16x8*)(wp + k + 32 * u);
#pragma unroll
      for (int i = 0; i < MT; ++i) af[i][u] = *(const bf16x8*)(ap[i] + k + 32 * u);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < MT; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[u], af[i][u], acc[i], 0, 0, 0);
  }
  for (; k < K; k += 32) {
    const bool ok = k + 8 * q < K;
    const bf16x8 wf = ok ? *(const bf16x8*)(wp + k) : bf16x8{};
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const bf16x8 af = ok ? *(const bf16x8*)(ap[i] + k) : bf16x8{};
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, af, acc[i], 0, 0, 0);
    }
  }
  // through LDS: whole 128-B row pieces out, the gate read the same way
#pragma unroll
  for (int i = 0; i < MT; ++i)
    *(uint2*)&tile[16 * i + r16][16 * w + 4 * q] = make_uint2(pack2bf(acc[i][0], acc[i][1]), pack2bf(acc[i][2], acc[i][3]));
  __syncthreads();
  const int c0 = blockIdx.x * 64;
  for (int e = threadIdx.x; e < 16 * MT * 8; e += 256) {
    const int r = e >> 3, c = (e & 7) * 8, t = t0 + r;
    if (t >= T || c0 + c >= N) continue;
    bf16_t* o = C + (long)t * ldc + b * sC + c0 + c;
    const bf16_t* gp = gate + (long)t * ldg + (long)b * N + c0 + c;
    if (vec) {
      uint4 v = *(const uint4*)&tile[r][c];
      if (gate) {
        float y[8], x[8];
        unpack8(v, y);
        unpack8(*(const uint4*)gp, x);
#pragma unroll
        for (int k = 0; k < 8; ++k) y[k] /= 1.f + __expf(-x[k]);
        v = pack8(y);
      }
      *(uint4*)o = v;
    } else {
      for (int k = 0; k < 8 && c0 + c + k < N; ++k) {
        const float y = bf2f(tile[r][c + k]);
        o[k] = f2bf(gate ? y / (1.f + __expf(-bf2f(gp[k]))) : y);
      }
    }
  }
}

// ---------------------------------------------------------------------------------------------
// absorbed attention over the pool, split over NP key partitions
// ---------------------------------------------------------------------------------------------
// Workgroup = (token, group of 16 NH heads, partition), 4 waves. Per 32-key tile (one LDS image, two
// buffers, LDS-DMA one tile ahead):
//   scores S^T = K Q^T (key on the MFMA row, head on the lane) by waves (key half, K-dim half) for
//   NH = 1 and (key half, head tile) for NH = 2; exchanged through LDS in accumulator layout;
//   every wave runs the same online softmax, packs P as the next MFMA's B operand, and accumulates
//   O^T += V^T P^T (head on the lane again) for its own quarter of the latent columns (V = the latent part of the same LDS image,
//   transposed reads). Two tiles' images are in flight or in use; three barriers per tile.
// A row's keys are cut in NP equal partitions (multiples of 32) from its own length, so a captured
// launch with a fixed NP balances every length. Image rows are CPR = 8 QS + 1 16-B chunks (odd: row
// reads conflict-free); chunks past KD repeat the row's last one.
struct DecArgs {
  const bf16_t* q;            // [T, H, KD]
  const bf16_t* pool; const int* tab; int max_pages, n_pages, n_rows;
  const int* row; const int* pos;
  float* part; float* ml;     // [T, H, NP, rank], [T, H, NP, 2] (max in log2 units, sum)
  int T, H, rank, KD, NP, HG;
  float scale_log2;
};

template <int QS, int RT, int NH>
__global__ __launch_bounds__(256, 2) void latent_decode_kernel(DecArgs a) {
  constexpr int CPR = 8 * QS + 1, ROWB = CPR * 16;
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
  const int hg = bid % a.HG, part = (bid / a.HG) % a.NP, t = bid / (a.HG * a.NP);
  const int h0 = hg * 16 * NH;
  // query fragments: lane holds Q[head r16][32 s + 8 g ..]
  const int kt = w & 1, hi = w >> 1;                 // key half; K-dim half (NH = 1) or head tile (NH = 2)
  const int qh = h0 + (NH == 2 ? hi * 16 : 0) + r16;
  const int sbase = NH == 1 ? hi * QS : 0;
  bf16x8 qf[QF];
  const bf16_t* qp = a.q + ((long)t * a.H + min(qh, a.H - 1)) * a.KD;  // heads past the last repeat it (not stored)
#pragma unroll
  for (int s = 0; s < QF; ++s) qf[s] = *(const bf16x8*)(qp + min(32 * (sbase + s) + 8 * g, a.KD - 8));
  const int row = min(max(a.row[t], 0), a.n_rows - 1);
  const int len = min(a.pos[t] + 1, a.max_pages * PAGE);
  const int per = ((len + a.NP - 1) / a.NP + 31) & ~31;
  const int k0 = part * per, k1 = min(len, k0 + per);
  if (k0 >= k1) {  // nothing for this partition (uniform over the workgroup)
    if (tid < 16 * NH && h0 + tid < a.H) {
      float* m = a.ml + (((long)t * a.H + h0 + tid) * a.NP + part) * 2;
      m[0] = -INFINITY;
      m[1] = 0.f;
    }
    return;
  }
  const int* tab = a.tab + (long)row * a.max_pages;

  // LDS-DMA sources: instruction j of wave w covers image chunks (4 j + w) * 64 + lane
  uint32_t src[NI];  // element offset from the tile's first cache row
#pragma unroll
  for (int j = 0; j < NI; ++j) {
    const int c = (4 * j + w) * 64 + lane;
    src[j] = (uint32_t)(min(c / CPR, 31) * a.KD + min(c % CPR * 8, a.KD - 8));
  }
  auto page_of = [&](int key0) { return min(max(tab[key0 / PAGE], 0), a.n_pages - 1); };
  auto stage = [&](int key0, int page, int buf) {
    const bf16_t* base = a.pool + ((long)page * PAGE + key0 % PAGE) * a.KD;
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
  stage(k0, page_of(k0), 0);
  if (k0 + 32 < k1) stage(k0 + 32, page_of(k0 + 32), 1);
  if (a.KD < 64 * QS) {  // columns past KD: zero in the query, anything finite in the image
#pragma unroll
    for (int s = 0; s < QF; ++s)
      if (32 * (sbase + s) + 8 * g >= a.KD) qf[s] = bf16x8{};
  }
#pragma unroll
  for (int s = 0; s < QF; ++s) asm volatile("" : "+v"(qf[s]));
  int buf = 0;
  for (int key0 = k0; key0 < k1; key0 += 32, buf ^= 1) {
    const bool n1 = key0 + 32 < k1, n2 = key0 + 64 < k1;
    const int page2 = n2 ? page_of(key0 + 64) : 0;
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
      }
      if (key0 + 32 > k1) {  // the row's last tile
#pragma unroll
        for (int k = 0; k < 2; ++k)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (key0 + 16 * k + 4 * g + i >= k1) s2[k][i] = -INFINITY;
      }
      float mx = fmaxf(fmaxf(fmaxf(s2[0][0], s2[0][1]), fmaxf(s2[0][2], s2[0][3])),
                       fmaxf(fmaxf(s2[1][0], s2[1][1]), fmaxf(s2[1][2], s2[1][3])));
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      // every tile holds a key of the row, so mn is finite; scale > 0 (launcher)
      const float mn = fmaxf(m[n], mx * a.scale_log2);
      const float alpha = fexp2(m[n] - mn);
      m[n] = mn;
      float rs = 0.f;
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = fexp2(fmaf(s2[k][i], a.scale_log2, -mn));
          s2[k][i] = p;
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
    // ---- O += P V: latent columns [16 RT w, 16 RT (w + 1)) ----
    const uint32_t va = lds_addr(img + (4 * g + ((lane >> 2) & 3)) * ROWB + w * RT * 32 + (lane & 3) * 8);
    rt_s16x4 v[2 * RT];
    if constexpr (RT == 8) ds_tr16_frag4<16 * ROWB, 32, 32 + 16 * ROWB>(va, va + 64, va + 128, va + 192, v);
    else if constexpr (RT == 4) ds_tr16_frag2<16 * ROWB, 32, 32 + 16 * ROWB>(va, va + 64, v);
    else ds_tr16_x4<16 * ROWB, 32, 32 + 16 * ROWB>(va, v[0], v[1], v[2], v[3]);
#pragma unroll
    for (int c = 0; c < RT; ++c) {
      const bf16x8 vf = cat4(v[2 * c], v[2 * c + 1]);
#pragma unroll
      for (int n = 0; n < NH; ++n) o[n][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pa[n], o[n][c], 0, 0, 0);
    }
    if (n2) {  // every wave is done with this image: the tile after the next one takes its place
      asm volatile("s_barrier" ::: "memory");
      stage(key0 + 64, page2, buf);
    }
  }
  // o[n][c][i]: head h0 + 16 n + r16, latent column 16 (RT w + c) + 4 g + i
#pragma unroll
  for (int n = 0; n < NH; ++n) {
    const int h = h0 + 16 * n + r16;
    if (h >= a.H) continue;
    const long th = ((long)t * a.H + h) * a.NP + part;
    float* po = a.part + th * a.rank + 16 * RT * w + 4 * g;
#pragma unroll
    for (int c = 0; c < RT; ++c)
      if (16 * (RT * w + c) + 4 * g < a.rank) *(f32x4*)(po + 16 * c) = o[n][c];  // rank % 8 == 0
    if (w == 0 && g == 0) *(float2*)(a.ml + th * 2) = make_float2(m[n], l[n]);
  }
}

// ---------------------------------------------------------------------------------------------
// segments of longer portions
// ---------------------------------------------------------------------------------------------
// out [kv rows of all segments, KD] = the cached rows of each segment, dense
template <typename V>
__global__ __launch_bounds__(256) void latent_gather_kernel(const V* __restrict__ pool, const int* __restrict__ tab,
                                                            int max_pages, int n_pages, const Seg* __restrict__ segs,
                                                            V* __restrict__ out, int vpr) {
  const Seg s = segs[blockIdx.y];
  const long n = (long)s.kv_len * vpr;
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long)gridDim.x * 256) {
    const int k = (int)(i / vpr), c = (int)(i % vpr);
    const int page = min(max(tab[(long)s.row * max_pages + min(k / PAGE, max_pages - 1)], 0), n_pages - 1);
    out[((long)s.kv_off + k) * vpr + c] = pool[((long)page * PAGE + k % PAGE) * vpr + c];
  }
}

// ---------------------------------------------------------------------------------------------
// flash attention of a portion over its request's expanded keys / values
// ---------------------------------------------------------------------------------------------
// The structure of attn_fwd_kernel (swapped S^T = K Q^T, P straight into the next MFMA, here O^T = V^T P^T; the double-
// buffered K / V tiles of 64 keys come by LDS-DMA, one barrier per tile): 128 query rows of one head per workgroup, 4 waves x
// 32 rows; a K row is [W_uk c (dim) | kr (rot)], padded to DQ columns; value width DV.
struct PreArgs {
  const bf16_t* q; long ldq;     // [tokens, ldq], head h at h * (dim + rot), rotated
  const bf16_t* kv; long ldk;    // expanded [kv rows, ldk]: unrotated keys at h * dim, values at v_col + h * vdim,
  int v_col, kr_col;             // the shared rotated key part at kr_col
  const float* sink;
  const bf16_t* gate; long ldg;
  bf16_t* o; long ldo;
  const Seg* segs; const int2* tiles; int n_tiles;   // {segment, first query row / 128}
  int H, dim, rot, vdim;
  float scale_log2;
};

template <int DQ, int DV>
__global__ __launch_bounds__(256, 2) void latent_prefill_kernel(PreArgs a) {
  constexpr int NQ = DQ / 8, NV = DV / 8, DS = DQ / 32, DT = DV / 16;
  constexpr int KB = 64 * DQ * 2, VB = 64 * DV * 2;
  constexpr int OROW = DV + 8;
  constexpr int TILES = 2 * (KB + VB), OB = 128 * OROW * 2;
  __shared__ __attribute__((aligned(16))) char smem[TILES > OB ? TILES : OB];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g = lane >> 4, r16 = lane & 15;
  const int lin = xcd_remap(blockIdx.x, gridDim.x);
  const int h = lin / a.n_tiles;
  const int2 tl = a.tiles[lin % a.n_tiles];
  const Seg sg = a.segs[tl.x];
  const int qblk0 = tl.y * 128, q0 = qblk0 + wid * 32;
  const int kend = min(sg.kv_len, sg.pos0 + min(qblk0 + 128, sg.q_len));
  const int hd = a.dim + a.rot;

  bf16x8 qf[2][DS];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int qr = min(q0 + 16 * u + r16, sg.q_len - 1);
    const bf16_t* qp = a.q + (long)(sg.q_off + qr) * a.ldq + (long)h * hd;
#pragma unroll
    for (int s = 0; s < DS; ++s) {
      const int c = 32 * s + 8 * g;
      qf[u][s] = c < hd ? *(const bf16x8*)(qp + c) : bf16x8{};
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
  // undoes the image's swizzle. Rows past the request's keys repeat the last one (masked); columns past the
  // head repeat its first chunk (the query is zero there, the values are not stored).
  constexpr int JK = KB / 4096, JV = VB / 4096;
  const bf16_t* kvb = a.kv + (long)sg.kv_off * a.ldk;
  auto chunk = [&](int j, bool v, int& key) -> int {  // key row and source column of the lane's chunk
    const int e = (4 * j + wid) * 64 + lane;
    key = v ? e / NV : e / NQ;
    const int c = 8 * (v ? vv_chunk<DV>(key, e % NV) : kq_chunk<DQ>(key, e % NQ));
    if (v) return a.v_col + h * a.vdim + (c < a.vdim ? c : 0);
    return c < a.dim ? h * a.dim + c : (c < hd ? a.kr_col + c - a.dim : h * a.dim);
  };
  uint32_t off[JK + JV];
#pragma unroll
  for (int j = 0; j < JK + JV; ++j) {
    int key;
    const int c = chunk(j < JK ? j : j - JK, j >= JK, key);
    off[j] = (uint32_t)key * (uint32_t)a.ldk + (uint32_t)c;
  }
  auto stage = [&](int kv0, int buf) {
    char* kd = smem + buf * (KB + VB);
    const bf16_t* base = kvb + (long)kv0 * a.ldk;
    auto issue = [&](int j, uint32_t o) {
      __builtin_amdgcn_global_load_lds((const void*)(base + o), (lds_void*)(kd + (j < JK ? 4 * j : KB / 1024 + 4 * (j - JK)) * 1024 +
                                                                            wid * 1024), 16, 0, 0);
    };
    if (kv0 + 64 <= sg.kv_len) {
#pragma unroll
      for (int j = 0; j < JK + JV; ++j) issue(j, off[j]);
    } else {  // the request's last tile
#pragma unroll
      for (int j = 0; j < JK + JV; ++j) {
        int key;
        const int c = chunk(j < JK ? j : j - JK, j >= JK, key);
        issue(j, (uint32_t)min(key, sg.kv_len - 1 - kv0) * (uint32_t)a.ldk + (uint32_t)c);
      }
    }
  };
  stage(0, 0);
  int cur = 0;
  for (int kv0 = 0; kv0 < kend; kv0 += 64, cur ^= 1) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this tile (issued one tile ago)
    asm volatile("s_barrier" ::: "memory");           // ... of every wave; the other buffer is free
    if (kv0 + 64 < kend) stage(kv0 + 64, cur ^ 1);
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
    if (!(kv0 + 63 <= sg.pos0 + q0 && kv0 + 63 < kend)) {  // the diagonal or the last tile
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int kk = kv0 + 16 * t + 4 * g + i;
            if (!(kk < kend && kk <= sg.pos0 + q0 + 16 * u + r16)) stt[t][u][i] = -INFINITY;
          }
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
      const float mn = fmaxf(m[u], mx * a.scale_log2);  // scale > 0 (launcher); key 0 keeps it finite
      alpha[u] = fexp2(m[u] - mn);
      m[u] = mn;
      float rs = 0.f;
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = fexp2(fmaf(stt[t][u][i], a.scale_log2, -mn));
          stt[t][u][i] = p;
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
      // the 4 transposed reads of two column tiles: keys + 0 / + 16, columns + 0 / + 16. The swizzle moves a
      // column tile by 32 B multiples that depend on the row, the same for rows 16 apart
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
  // the sink joins the denominator; O through LDS, gated on the way out
  const float sink2 = a.sink[h] * 1.4426950408889634f;
  bf16_t* Os = (bf16_t*)smem;
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const float M = fmaxf(m[u], sink2);
    const float f = exp2f(m[u] - M);
    const float sc = f / (l[u] * f + exp2f(sink2 - M));
    const int r = wid * 32 + 16 * u + r16;
#pragma unroll
    for (int c = 0; c < DT; ++c)
      *(uint2*)(Os + r * OROW + 16 * c + 4 * g) =
          make_uint2(pack2bf(o[u][c][0] * sc, o[u][c][1] * sc), pack2bf(o[u][c][2] * sc, o[u][c][3] * sc));
  }
  __syncthreads();
  for (int e = tid; e < 128 * NV; e += 256) {
    const int r = e / NV, c = (e % NV) * 8;
    if (qblk0 + r < sg.q_len && c < a.vdim) {
      const long tok = sg.q_off + qblk0 + r;
      float v[8], x[8];
      unpack8(*(const uint4*)(Os + r * OROW + c), v);
      unpack8(*(const uint4*)(a.gate + tok * a.ldg + (long)h * a.vdim + c), x);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[k] = v[k] / (1.f + __expf(-x[k]));
      *(uint4*)(a.o + tok * a.ldo + (long)h * a.vdim + c) = pack8(v);
    }
  }
}

// ---------------------------------------------------------------------------------------------
// absorbed attention of any size and type: one workgroup per (token, head), 256 keys at a time
// ---------------------------------------------------------------------------------------------
struct LatAnyArgs {
  const void* q; const void* pool; const int* tab; int max_pages, n_pages, n_rows;
  const int* row; const int* pos;
  const float* sink;
  void* o;                     // [T, H, rank] latent outputs (softmax with the sink applied)
  int H, rank, KD;
  float scale;
};

template <typename T>
__global__ __launch_bounds__(256) void latent_any_kernel(LatAnyArgs a) {
  extern __shared__ float sm[];  // q [KD], acc [rank], p [256], sbuf [4]
  float* qs = sm;
  float* acc = qs + a.KD;
  float* ps = acc + a.rank;
  float* sbuf = ps + 256;
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x;
  const int row = min(max(a.row[t], 0), a.n_rows - 1);
  const int len = min(a.pos[t] + 1, a.max_pages * PAGE);
  const int* tab = a.tab + (long)row * a.max_pages;
  for (int c = tid; c < a.KD; c += 256) qs[c] = ld((const T*)a.q + ((long)t * a.H + h) * a.KD + c);
  for (int c = tid; c < a.rank; c += 256) acc[c] = 0.f;
  float m = a.sink[h], l = 1.f;  // the sink: exp(sink - m) = 1
  __syncthreads();
  for (int k0 = 0; k0 < len; k0 += 256) {
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key < len) {
      const int page = min(max(tab[key / PAGE], 0), a.n_pages - 1);
      const T* kp = (const T*)a.pool + ((long)page * PAGE + key % PAGE) * a.KD;
      float d = 0.f;
      for (int c = 0; c < a.KD; ++c) d = fmaf(qs[c], ld(kp + c), d);
      s = d * a.scale;
    }
    const float mn = fmaxf(m, block_max(s, sbuf));
    const float alpha = expf(m - mn);
    const float p = key < len ? expf(s - mn) : 0.f;
    ps[tid] = p;
    l = l * alpha + block_sum(p, sbuf);
    m = mn;
    __syncthreads();
    const int n = min(256, len - k0);
    for (int c = tid; c < a.rank; c += 256) {
      float y = acc[c] * alpha;
      for (int k = 0; k < n; ++k) {
        const int kk = k0 + k;
        const int page = min(max(tab[kk / PAGE], 0), a.n_pages - 1);
        y = fmaf(ps[k], ld((const T*)a.pool + ((long)page * PAGE + kk % PAGE) * a.KD + c), y);
      }
      acc[c] = y;
    }
    __syncthreads();
  }
  for (int c = tid; c < a.rank; c += 256) st((T*)a.o + ((long)t * a.H + h) * a.rank + c, acc[c] / l);
}

}  // namespace la
}  // namespace rt

using namespace rt;
using namespace rt::la;

extern "C" int rt_latent_prep(int f32, void* proj, long ldp, int kv_col, const void* norm_w, float eps,
                              const float* cosT, const float* sinT, int max_pos, int rdims, const int* row,
                              const int* pos, void* pool, const int* tab, int max_pages, int n_pages, int n_rows,
                              void* qabs, int n_abs, int T, int H, int dim, int rot, int rank, hipStream_t stream) {
  if (T <= 0) return 0;
  if (rot % 2 || rdims % 2 || rdims > rot) return -1;
  PrepArgs a{proj, ldp, kv_col, norm_w, eps, cosT, sinT, max_pos, rdims, row, pos, pool, tab, max_pages, n_pages,
             n_rows, qabs, n_abs, H, dim, rot, rank, 0};
  a.vec = rdims == rot && rot % 8 == 0 && dim % 8 == 0 && rank % 8 == 0 && ldp % 8 == 0 && (uintptr_t)proj % 16 == 0;
  if (f32) hipLaunchKernelGGL((latent_prep_kernel<float>), dim3(T), dim3(256), 0, stream, a);
  else hipLaunchKernelGGL((latent_prep_kernel<bf16_t>), dim3(T), dim3(256), 0, stream, a);
  RT_LAUNCH_CHECK();
  return 0;
}

// bf16, K % 8 == 0, 16-B aligned rows
extern "C" int rt_head_gemm(const void* A, long lda, long sA, const void* W, long ldw, long sW, void* C, long ldc,
                            long sC, int T, int N, int K, int batch, const void* gate, long ldg,
                            hipStream_t stream) {
  if (T <= 0 || N <= 0 || batch <= 0) return 0;
  if (K % 8 || lda % 8 || sA % 8 || ldw % 8 || sW % 8 || batch > 65535 || (T + 15) / 16 > 65535) return -1;
  const int mt = T > 128 ? 4 : 1;
  // 16-B output pieces (and gate reads)
  const int vec = N % 8 == 0 && ldc % 8 == 0 && sC % 8 == 0 && (uintptr_t)C % 16 == 0 &&
                  (!gate || (ldg % 8 == 0 && (uintptr_t)gate % 16 == 0));
  dim3 grid((N + 63) / 64, batch, (T + 16 * mt - 1) / (16 * mt));
#define HG_(M) hipLaunchKernelGGL(head_gemm_kernel<M>, grid, dim3(256), 0, stream, (const bf16_t*)A, lda, sA, (const bf16_t*)W, \
                                  ldw, sW, (bf16_t*)C, ldc, sC, T, N, K, (const bf16_t*)gate, ldg, vec)
  if (mt == 4) HG_(4); else HG_(1);
#undef HG_
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_latent_decode_ok(int rank, int KD) {
  return rank % 8 == 0 && KD % 8 == 0 && rank <= 512 && KD <= 640 && (rank > 256 || KD <= 384) && (rank > 128 || KD <= 256);
}

extern "C" int rt_latent_decode(const void* q, const void* pool, const int* tab, int max_pages, int n_pages, int n_rows,
                                const int* row, const int* pos, float* part, float* ml, int T, int H, int rank, int KD,
                                int NP, float scale, hipStream_t stream) {
  if (T <= 0) return 0;
  if (!rt_latent_decode_ok(rank, KD) || NP < 1 || !(scale > 0)) return -1;
  const int NH = H > 16 ? 2 : 1;
  const int HG = (H + 16 * NH - 1) / (16 * NH);
  DecArgs a{(const bf16_t*)q, (const bf16_t*)pool, tab, max_pages, n_pages, n_rows, row, pos, part, ml, T, H, rank, KD,
            NP, HG, scale * 1.4426950408889634f};
  dim3 grid((unsigned)((long)T * HG * NP)), block(256);
#define LD_(QS, RT)                                                                                       \
  do {                                                                                                    \
    if (NH == 1) hipLaunchKernelGGL((latent_decode_kernel<QS, RT, 1>), grid, block, 0, stream, a);        \
    else hipLaunchKernelGGL((latent_decode_kernel<QS, RT, 2>), grid, block, 0, stream, a);                \
  } while (0)
  if (rank <= 128) {
    if (KD <= 192) LD_(3, 2); else LD_(4, 2);
  } else if (rank <= 256) {
    if (KD <= 320) LD_(5, 4); else LD_(6, 4);
  } else {
    if (KD <= 576) LD_(9, 8); else LD_(10, 8);
  }
#undef LD_
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_latent_gather(int f32, const void* pool, const int* tab, int max_pages, int n_pages, const void* segs,
                                int n_segs, int max_kv, void* out, int KD, hipStream_t stream) {
  if (n_segs <= 0 || max_kv <= 0) return 0;
  if (n_segs > 65535) return -1;
  const int bytes = KD * (f32 ? 4 : 2);
  const int vb = bytes % 16 == 0 ? 16 : 2;
  const int vpr = bytes / vb;
  const long n = (long)max_kv * vpr;
  dim3 grid((unsigned)std::min<long>((n + 255) / 256, 4096), n_segs);
  if (vb == 16)
    hipLaunchKernelGGL((latent_gather_kernel<u32x4>), grid, dim3(256), 0, stream, (const u32x4*)pool, tab, max_pages,
                       n_pages, (const Seg*)segs, (u32x4*)out, vpr);
  else
    hipLaunchKernelGGL((latent_gather_kernel<uint16_t>), grid, dim3(256), 0, stream, (const uint16_t*)pool, tab,
                       max_pages, n_pages, (const Seg*)segs, (uint16_t*)out, vpr);
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_latent_prefill_ok(int dim, int rot, int vdim) {
  return dim % 8 == 0 && rot % 8 == 0 && vdim % 8 == 0 && dim + rot <= 256 && vdim <= 128;
}

extern "C" int rt_latent_prefill(const void* q, long ldq, const void* kv, long ldk, int v_col, int kr_col,
                                 const float* sink, const void* gate, long ldg, void* o, long ldo, const void* segs,
                                 const void* tiles, int n_tiles, int H, int dim, int rot, int vdim, float scale,
                                 hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  if (!(scale > 0) || !rt_latent_prefill_ok(dim, rot, vdim) || ldq % 8 || ldk % 8 || v_col % 8 || kr_col % 8 || ldg % 8 || ldo % 8) return -1;
  PreArgs a{(const bf16_t*)q, ldq, (const bf16_t*)kv, ldk, v_col, kr_col, sink, (const bf16_t*)gate, ldg,
            (bf16_t*)o, ldo, (const Seg*)segs, (const int2*)tiles, n_tiles, H, dim, rot, vdim,
            scale * 1.4426950408889634f};
  dim3 grid((unsigned)((long)n_tiles * H)), block(256);
  const int dq = dim + rot;
#define LP_(DQ)                                                                                         \
  do {                                                                                                  \
    if (vdim <= 64) hipLaunchKernelGGL((latent_prefill_kernel<DQ, 64>), grid, block, 0, stream, a);     \
    else hipLaunchKernelGGL((latent_prefill_kernel<DQ, 128>), grid, block, 0, stream, a);               \
  } while (0)
  if (dq <= 64) LP_(64);
  else if (dq <= 128) LP_(128);
  else if (dq <= 192) LP_(192);
  else LP_(256);
#undef LP_
  RT_LAUNCH_CHECK();
  return 0;
}

extern "C" int rt_latent_any(int f32, const void* q, const void* pool, const int* tab, int max_pages, int n_pages,
                             int n_rows, const int* row, const int* pos, const float* sink, void* o, int T, int H,
                             int rank, int KD, float scale, hipStream_t stream) {
  if (T <= 0) return 0;
  if (T > 65535) return -1;
  const size_t lds = (size_t)(KD + rank + 256 + 4) * 4;
  if (lds > 65536) return -2;
  LatAnyArgs a{q, pool, tab, max_pages, n_pages, n_rows, row, pos, sink, o, H, rank, KD, scale};
  if (f32) hipLaunchKernelGGL((latent_any_kernel<float>), dim3(H, T), dim3(256), lds, stream, a);
  else hipLaunchKernelGGL((latent_any_kernel<bf16_t>), dim3(H, T), dim3(256), lds, stream, a);
  RT_LAUNCH_CHECK();
  return 0;
}
