// Gated delta rule for gfx950. Per sequence and head a state S [D, V] (fp32):
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// q, k (per key head, shared by H / K heads), v: projections through a causal convolution of `taps` and silu;
// q, k then unit vectors, q times D^-1/2; beta = sigmoid(b); g = exp(-exp(A) softplus(a + dt)) per head or
// per key channel; the read-out is RMS-normed over V, weighted and gated (silu or sigmoid of z). Everything
// behind the convolutions is fp32, for models of either type.
//
// State of a request (cache row): S [H, D, V] fp32 and a ring of the last projections [taps][C] (C = q | k | v
// channels; position p at slot p % taps). At position 0 both count as zero, whatever they hold, so a slot
// that is used again needs no clearing. Rows < 0 (parked) read zeros and write nothing.
//
//   delta_step    one token per request: everything in one kernel, the state read and written once
//   portions:     delta_prep (chunks of 16 tokens, all in parallel) -> delta_scan (chunks in order, fp32 MFMA;
//                 value columns in parallel) -> delta_out (norm, gate), delta_commit (ring)
//
// Chunk form (tokens 1..16 of a chunk, G_i = summed log decays, S0 = state ahead of it):
//   A_ij = beta_i sum_d k_id k_jd e^(G_id - G_jd)  (j < i),  P_ij = sum_d q_id k_jd e^(G_id - G_jd)  (j <= i)
//   U = T (V - (k e^G) S0) with T = (I + A)^-1 diag(beta);  O = (q e^G) S0 + P U
//   S = diag(e^G_16) S0 + (k e^(G_16 - G))^T U
// Every exponent is <= 0: A and P are built per level of a binary split (rows of an upper half against columns
// of its lower half, both scaled to the last row of the lower half).
#include "rt_common.h"

#include <algorithm>

namespace rt {
namespace dr {

constexpr int CH = 16;  // tokens per chunk

template <typename T> __device__ __forceinline__ float ld(const T* p);
template <> __device__ __forceinline__ float ld<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ld<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void st(T* p, float v);
template <> __device__ __forceinline__ void st<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void st<float>(float* p, float v) { *p = v; }

// N floats, aligned to 16 bytes from four on
template <int N>
__device__ __forceinline__ void ldf(const float* p, float* o) {
  if constexpr (N % 4 == 0) {
#pragma unroll
    for (int k = 0; k < N; k += 4) *(f32x4*)(o + k) = *(const f32x4*)(p + k);
  } else {
    o[0] = p[0];
  }
}
template <int N>
__device__ __forceinline__ void stf(float* p, const float* o) { ldf<N>(o, p); }

__device__ __forceinline__ float sigmoid(float x) { return __builtin_amdgcn_rcpf(1.f + expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float gate_of(float z, bool silu) { return (silu ? z : 1.f) * sigmoid(z); }

struct Args {
  const void* x; long ldx;            // [N, ldx] projections: q | k | v channels contiguous at column 0 of x
  const void* b; long ldb;            // [N, H]
  const void* a; long lda;            // [N, H] or (channel) [N, H * D]
  const void* z; long ldz;            // [N, H * V]
  const void* conv;                   // [C, taps]
  const float* A_log; const float* dt;  // [H], [H] or (channel) [H * D]
  const void* norm_w; float eps;      // [V]
  const int* row; const int* pos;     // per token
  float* S; void* ring; int n_rows;
  void* out; long ldo; float out_scale;  // [N, H * V]
  int H, K, D, V, taps, channel, silu;
};

// channels of the short convolutions: one output, the token's input from x, older ones from x or the ring
template <typename T>
struct Conv {
  const Args& a;
  const T* x;      // the run's first token, at the convolution's channels
  const T* ring;   // the row's ring (null: nothing before the run)
  int start, C;    // position of the run's first token
  __device__ __forceinline__ float raw(int p, int c) const {
    if (p >= start) return ld(x + (long)(p - start) * a.ldx + c);
    return ring && p >= 0 ? ld(ring + (long)(p % a.taps) * C + c) : 0.f;
  }
  __device__ __forceinline__ float operator()(int p, int c) const {
    const T* w = (const T*)a.conv + (long)c * a.taps;
    float y = 0.f;
    for (int j = 0; j < a.taps; ++j) y = fmaf(ld(w + j), raw(p - (a.taps - 1 - j), c), y);
    return y * sigmoid(y);
  }
};

// ---------------------------------------------------------------------------------------------
// one token per request. Thread = VEC value columns x NR key rows of the state, held in registers. The small inputs are
// on their way first (as the words they lie in memory as: a conversion would wait for them), then the state; the
// projections' part (convolutions, unit norms, decays) runs meanwhile.
// ---------------------------------------------------------------------------------------------
template <typename T> __device__ __forceinline__ uint32_t word(const T* p);
template <> __device__ __forceinline__ uint32_t word<bf16_t>(const bf16_t* p) { return *p; }
template <> __device__ __forceinline__ uint32_t word<float>(const float* p) { return __float_as_uint(*p); }
template <typename T> __device__ __forceinline__ float value(uint32_t w) { return __uint_as_float(sizeof(T) == 2 ? w << 16 : w); }

template <typename T, int VEC, int NR, int BLOCK>
__global__ __launch_bounds__(BLOCK) void delta_step_kernel(Args a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];  // sums [2][RG][V]; k, q, g [D]; v, o [V]
  constexpr int PRE = 2, TAP = 4;  // channels per thread and their last taps that are loaded ahead
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int D = a.D, V = a.V, taps = a.taps, kh = h / (a.H / a.K);
  const int ncol = (V + VEC - 1) / VEC, RG = BLOCK / ncol;
  float* sum = sm;
  float* ks = sum + 2 * RG * V;
  float* qs = ks + D;
  float* gs = qs + D;
  float* vs = gs + D;
  float* os = vs + V;
  const int row_ = a.row[t], pos = max(a.pos[t], 0);
  const bool live = row_ >= 0 && row_ < a.n_rows, carry = live && pos > 0;
  const int row = live ? row_ : 0;
  const int cg = tid % ncol, rg = tid / ncol;
  const bool mine = rg < RG;
  const int KD = a.K * D, C = 2 * KD + a.H * V, nch = 2 * D + V, slot = pos % taps;
  const T* xt = (const T*)a.x + (long)t * a.ldx;
  const T* conv = (const T*)a.conv;
  T* ring = (T*)a.ring + (long)row * taps * C;
  auto chan = [&](int i) { return i < D ? kh * D + i : (i < 2 * D ? KD + kh * D + i - D : 2 * KD + h * V + i - 2 * D); };
  auto past = [&](int c, int back) {  // the channel's input `back` < taps tokens ago (a finite or stale word: see seen)
    int s = slot - back;
    if (s < 0) s += taps;
    return word(back ? ring + (long)s * C + c : xt + c);
  };
  auto seen = [&](int back) { return back < taps && (back == 0 || (carry && pos >= back)); };
  uint32_t xw[PRE][TAP], ww[PRE][TAP];
#pragma unroll
  for (int k = 0; k < PRE; ++k) {
    const int c = chan(min(tid + k * BLOCK, nch - 1));
#pragma unroll
    for (int j = 0; j < TAP; ++j) {
      const int back = min(j, taps - 1);
      xw[k][j] = past(c, back);
      ww[k][j] = word(conv + (long)c * taps + taps - 1 - back);
    }
  }
  const T* ap = (const T*)a.a + (long)t * a.lda + (a.channel ? (long)h * D + min(tid, D - 1) : h);
  const uint32_t aw = word(ap), bw = word((const T*)a.b + (long)t * a.ldb + h);
  const float dt = a.dt[a.channel ? (long)h * D + min(tid, D - 1) : h], A_log = a.A_log[h];
  const T* zp = (const T*)a.z + (long)t * a.ldz + (long)h * V;
  const uint32_t zw = word(zp + min(tid, V - 1)), nw = word((const T*)a.norm_w + min(tid, V - 1));
  asm volatile("" ::: "memory");
  float* Sp = a.S + (((long)row * a.H + h) * D) * V + (mine ? cg * VEC : 0);
  float s[NR][VEC];
#pragma unroll
  for (int j = 0; j < NR; ++j)
#pragma unroll
    for (int e = 0; e < VEC; ++e) s[j][e] = 0.f;
  if (carry) {  // threads and rows past the edge repeat the last row; they take no part below
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const float* p = Sp + (long)min(rg + j * RG, D - 1) * V;
      if constexpr (VEC == 4) {
        const float4 v = *(const float4*)p;
        s[j][0] = v.x; s[j][1] = v.y; s[j][2] = v.z; s[j][3] = v.w;
      } else {
        s[j][0] = *p;
      }
    }
  }
  auto put = [&](int i, int c, float y) {
    y *= sigmoid(y);
    (i < D ? qs[i] : (i < 2 * D ? ks[i - D] : vs[i - 2 * D])) = y;
    // the slot of this position is read by nobody at this position; heads that share a key head share the write
    if (live && (i >= 2 * D || h % (a.H / a.K) == 0)) ring[(long)slot * C + c] = xt[c];
  };
  auto older = [&](int c, int j0) {  // taps from j0 tokens ago on
    float y = 0.f;
    for (int j = taps - 1; j >= j0; --j)
      if (seen(j)) y = fmaf(ld(conv + (long)c * taps + taps - 1 - j), value<T>(past(c, j)), y);
    return y;
  };
#pragma unroll
  for (int k = 0; k < PRE; ++k) {
    const int i = tid + k * BLOCK;
    if (i >= nch) continue;
    const int c = chan(i);
    float y = older(c, TAP);
#pragma unroll
    for (int j = TAP - 1; j >= 0; --j) y = seen(j) ? fmaf(value<T>(ww[k][j]), value<T>(xw[k][j]), y) : y;
    put(i, c, y);
  }
  for (int i = tid + PRE * BLOCK; i < nch; i += BLOCK) put(i, chan(i), older(chan(i), 0));
  const float A = expf(A_log);
  if (a.channel) {
    if (tid < D) gs[tid] = expf(-A * softplus(value<T>(aw) + dt));
    for (int d = tid + BLOCK; d < D; d += BLOCK)
      gs[d] = expf(-A * softplus(ld((const T*)a.a + (long)t * a.lda + (long)h * D + d) + a.dt[(long)h * D + d]));
  } else {
    const float g = expf(-A * softplus(value<T>(aw) + dt));
    for (int d = tid; d < D; d += BLOCK) gs[d] = g;
  }
  __syncthreads();
  float qq = 0.f, kk = 0.f, qk = 0.f;  // every wave for itself
  for (int d = lane; d < D; d += 64) {
    qq += qs[d] * qs[d];
    kk += ks[d] * ks[d];
    qk += qs[d] * ks[d];
  }
  const float iq = 1.f / sqrtf(wave_sum(qq) + 1e-6f) / sqrtf((float)D), ik = 1.f / sqrtf(wave_sum(kk) + 1e-6f);
  qk = wave_sum(qk) * iq * ik;
  const float beta = sigmoid(value<T>(bw));
  __attribute__((aligned(16))) float pk[VEC], pq[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) { pk[e] = 0.f; pq[e] = 0.f; }
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    const int d = rg + j * RG;
    if (mine && d < D) {
      const float g = gs[d], k = ks[d] * ik, q = qs[d] * iq;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        s[j][e] *= g;
        pk[e] = fmaf(k, s[j][e], pk[e]);
        pq[e] = fmaf(q, s[j][e], pq[e]);
      }
    }
  }
  if (mine) {
    stf<VEC>(sum + rg * V + cg * VEC, pk);
    stf<VEC>(sum + (RG + rg) * V + cg * VEC, pq);
  }
  __syncthreads();
  float u[VEC];
  if (mine) {
    __attribute__((aligned(16))) float sk[VEC], sq[VEC], x[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) { sk[e] = 0.f; sq[e] = 0.f; }
#pragma unroll 4
    for (int r = 0; r < RG; ++r) {
      ldf<VEC>(sum + r * V + cg * VEC, x);
#pragma unroll
      for (int e = 0; e < VEC; ++e) sk[e] += x[e];
      if (rg == 0) {
        ldf<VEC>(sum + (RG + r) * V + cg * VEC, x);
#pragma unroll
        for (int e = 0; e < VEC; ++e) sq[e] += x[e];
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      u[e] = beta * (vs[cg * VEC + e] - sk[e]);
      if (rg == 0) os[cg * VEC + e] = fmaf(qk, u[e], sq[e]);  // S^T q behind the write
    }
    if (live) {
#pragma unroll
      for (int j = 0; j < NR; ++j) {
        const int d = rg + j * RG;
        if (d < D) {
          const float k = ks[d] * ik;
#pragma unroll
          for (int e = 0; e < VEC; ++e) s[j][e] = fmaf(k, u[e], s[j][e]);
          if constexpr (VEC == 4) *(float4*)(Sp + (long)d * V) = make_float4(s[j][0], s[j][1], s[j][2], s[j][3]);
          else Sp[(long)d * V] = s[j][0];
        }
      }
    }
  }
  __syncthreads();
  float oo = 0.f;
  for (int c = lane; c < V; c += 64) oo += os[c] * os[c];
  const float r = a.out_scale / sqrtf(wave_sum(oo) / V + a.eps);
  T* out = (T*)a.out + (long)t * a.ldo + (long)h * V;
  if (tid < V) st(out + tid, os[tid] * r * value<T>(nw) * gate_of(value<T>(zw), a.silu));
  for (int c = tid + BLOCK; c < V; c += BLOCK) st(out + c, os[c] * r * ld((const T*)a.norm_w + c) * gate_of(ld(zp + c), a.silu));
}

// ---------------------------------------------------------------------------------------------
// portions
// ---------------------------------------------------------------------------------------------
// runs: {row, first token, tokens, position of the first}; chunks: {run, chunk of the run}, a run's chunks
// consecutive. Workspace per (chunk, head): k e^G, q e^G [CH][DP], k e^(G_16 - G) transposed [DP][CH], e^G_16 [DP],
// T, P [CH][CH] floats, the matrices as the MFMA's first operand: row m, column 16 r + 4 g + i of a [CH][..] one (of
// rows 16 r + m, column 4 g + i of the transposed one) is element (r * 64 + 16 g + m) * 4 + i, so a wave loads 1 KB runs.
struct Work {
  const int4* runs; const int2* chunks;
  float* ws;    // a head's chunks side by side
  int n_chunks, chunk0;
  long ldv;
  void* v;      // [N, ldv] convolved values, rows of the batch's tokens; ldv = H * V, even
  float* o;     // [N, H * V] read-outs
};
template <int DP> struct Lay {
  static __device__ __forceinline__ int sq(int row, int col) { return (16 * (col >> 2) + row) * 4 + (col & 3); }  // T, P
  static constexpr int KT = 0, QT = CH * DP, KE = 2 * CH * DP, EG = 3 * CH * DP, T = EG + DP, P = T + CH * CH, N = P + CH * CH;
};

// N consecutive elements: 8 bf16 or 4 floats (16 bytes, aligned), or 1
template <typename T, int N>
__device__ __forceinline__ void ldn(const T* p, float* o) {
  if constexpr (N == 8) unpack8(*(const uint4*)p, o);
  else if constexpr (N == 4) *(f32x4*)o = *(const f32x4*)p;
  else o[0] = ld(p);
}
template <typename T, int N>
__device__ __forceinline__ void stn(T* p, const float* o) {
  if constexpr (N == 8) *(uint4*)p = pack8(o);
  else if constexpr (N == 4) *(f32x4*)p = *(const f32x4*)o;
  else st(p, o[0]);
}

// convolution and silu of channels c .. c + N - 1 at positions p .. p + 3, zeros from position p + n on. TAPS: their
// number (every load issued ahead), 0: any
template <typename T, int N, int TAPS>
__device__ __forceinline__ void conv4(const Conv<T>& cv, int p, int n, int c, float (&y)[4][N]) {
  const int taps = TAPS ? TAPS : cv.a.taps;
  const T* w = (const T*)cv.a.conv + (long)c * taps;
  // a row that counts as zero stays unread
  auto row = [&](int q, float (&v)[N]) {
    const T* src = q >= cv.start ? cv.x + (long)(q - cv.start) * cv.a.ldx : cv.ring + (long)(max(q, 0) % taps) * cv.C;
#pragma unroll
    for (int e = 0; e < N; ++e) v[e] = 0.f;
    if (q < p + n && (q >= cv.start || (cv.ring && q >= 0))) ldn<T, N>(src + c, v);
  };
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < N; ++e) y[i][e] = 0.f;
  if constexpr (TAPS > 0) {
    __attribute__((aligned(16))) float v[TAPS + 3][N], f[TAPS][N];  // f: the weights as they lie, [channel][tap]
#pragma unroll
    for (int j = 0; j < TAPS + 3; ++j) row(p - (TAPS - 1) + j, v[j]);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) ldn<T, N>(w + j * N, f[j]);
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < N; ++e) y[i][e] = fmaf((&f[0][0])[e * TAPS + j], v[i + j][e], y[i][e]);
  } else {
    for (int j = 0; j < taps; ++j) {
      float wj[N];
#pragma unroll
      for (int e = 0; e < N; ++e) wj[e] = ld(w + e * taps + j);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        __attribute__((aligned(16))) float v[N];
        row(p + i - (taps - 1 - j), v);
#pragma unroll
        for (int e = 0; e < N; ++e) y[i][e] = fmaf(wj[e], v[e], y[i][e]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < N; ++e) y[i][e] = i < n ? y[i][e] * sigmoid(y[i][e]) : 0.f;
}

// workgroup = (head, chunk); CHN: a decay per key channel, else per head. N: elements per access
template <typename T, int DP, bool CHN, int N, int TAPS>
__global__ __launch_bounds__(256) void delta_prep_kernel(Args a, Work w) {
  constexpr int LD = DP + 4, R = DP / 16;
  using L = Lay<DP>;
  __shared__ __attribute__((aligned(16))) float kx[CH][LD], qx[CH][LD], G[CHN ? CH : 1][LD];
  __shared__ float As[CH][CH + 1], Ps[CH][CH + 1], beta[CH], dot[CH], Gs[CH];
  __shared__ f32x4 red[CHN ? 1 : 3][2][64];
  const int h = blockIdx.x, ci = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int2 ck = w.chunks[ci];
  const int4 run = w.runs[ck.x];
  const int n = min(CH, run.z - ck.y * CH), p0 = run.w + ck.y * CH, t0 = run.y + ck.y * CH;
  const int D = a.D, V = a.V, kh = h / (a.H / a.K), KD = a.K * D, C = 2 * KD + a.H * V;
  const bool carry = run.x >= 0 && run.x < a.n_rows && run.w > 0;
  const Conv<T> conv{a, (const T*)a.x + (long)run.y * a.ldx,
                     carry ? (const T*)a.ring + (long)run.x * a.taps * C : nullptr, run.w, C};
  const float A = expf(a.A_log[h]);
  if (tid < CH) {
    const T* bp = (const T*)a.b + (long)(t0 + tid) * a.ldb + h;
    beta[tid] = tid < n ? sigmoid(ld(bp)) : 0.f;
    if constexpr (!CHN) {  // summed log decays
      float g = tid < n ? -A * softplus(ld((const T*)a.a + (long)(t0 + tid) * a.lda + h) + a.dt[h]) : 0.f;
#pragma unroll
      for (int o = 1; o < CH; o *= 2) {
        const float up = __shfl_up(g, o, CH);
        if (tid >= o) g += up;
      }
      Gs[tid] = g;
    }
  }
  const int gd = D / N, gv = V / N, ng = 2 * gd + gv;
  for (int e = tid; e < 4 * ng; e += 256) {  // four tokens of N channels
    const int i0 = e / ng * 4, gr = e % ng;
    const int c = gr < gd ? kh * D + gr * N : (gr < 2 * gd ? KD + kh * D + (gr - gd) * N : 2 * KD + h * V + (gr - 2 * gd) * N);
    __attribute__((aligned(16))) float y[4][N];
    conv4<T, N, TAPS>(conv, p0 + i0, n - i0, c, y);
    if (gr >= 2 * gd) {
      T* v = (T*)w.v + (long)(t0 + i0) * w.ldv + (c - 2 * KD);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (i0 + i < n) stn<T, N>(v + i * w.ldv, y[i]);
    } else {
      float* x = gr < gd ? &qx[i0][gr * N] : &kx[i0][(gr - gd) * N];
#pragma unroll
      for (int i = 0; i < 4; ++i) stf<N>(x + i * LD, y[i]);
    }
  }
  if (D < DP)
    for (int e = tid; e < CH * (DP - D); e += 256) {
      const int i = e / (DP - D), d = D + e % (DP - D);
      kx[i][d] = 0.f;
      qx[i][d] = 0.f;
      if constexpr (CHN) G[i][d] = 0.f;
    }
  if constexpr (CHN) {
    for (int e = tid; e < CH * gd; e += 256) {
      const int i = e / gd, d = e % gd * N;
      __attribute__((aligned(16))) float v[N];
#pragma unroll
      for (int k = 0; k < N; ++k) v[k] = 0.f;
      if (i < n) {
        ldn<T, N>((const T*)a.a + (long)(t0 + i) * a.lda + (long)h * D + d, v);
#pragma unroll
        for (int k = 0; k < N; ++k) v[k] = -A * softplus(v[k] + a.dt[(long)h * D + d + k]);
      }
      stf<N>(&G[i][d], v);
    }
  }
  __syncthreads();
  {  // unit vectors: 16 threads per token
    const int i = tid >> 4;
    float kk = 0.f, qq = 0.f, qk = 0.f;
    for (int d = 4 * (tid & 15); d < DP; d += 64) {
      const f32x4 k4 = *(const f32x4*)&kx[i][d], q4 = *(const f32x4*)&qx[i][d];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        kk = fmaf(k4[j], k4[j], kk);
        qq = fmaf(q4[j], q4[j], qq);
        qk = fmaf(q4[j], k4[j], qk);
      }
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) {
      kk += __shfl_xor(kk, o, 64);
      qq += __shfl_xor(qq, o, 64);
      qk += __shfl_xor(qk, o, 64);
    }
    const float ik = 1.f / sqrtf(kk + 1e-6f), iq = 1.f / sqrtf(qq + 1e-6f) / sqrtf((float)D);
    for (int d = 4 * (tid & 15); d < DP; d += 64) {
      *(f32x4*)&kx[i][d] *= ik;
      *(f32x4*)&qx[i][d] *= iq;
    }
    if ((tid & 15) == 0) dot[i] = qk * ik * iq;
  }
  if constexpr (CHN) {
    for (int d = tid; d < DP; d += 256) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        s += G[i][d];
        G[i][d] = s;
      }
    }
  }
  __syncthreads();
  float* ws = w.ws + ((long)h * w.n_chunks + w.chunk0 + ci) * L::N;
  const int m = lane & 15, g = lane >> 4;
  f32x4 ka = {0.f, 0.f, 0.f, 0.f}, pa = {0.f, 0.f, 0.f, 0.f};
  if constexpr (CHN) {  // A and P: wave = level of the split, half size s
    const int s = 8 >> wid, piv = (m & ~(2 * s - 1)) + s - 1;
#pragma unroll 2
    for (int r = 0; r < R; ++r) {
      const int d = 16 * r + 4 * g;
      const f32x4 k4 = *(const f32x4*)&kx[m][d], q4 = *(const f32x4*)&qx[m][d];
      const f32x4 g4 = *(const f32x4*)&G[m][d], v4 = *(const f32x4*)&G[piv][d];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float e = expf(-fabsf(g4[i] - v4[i]));
        const float x = k4[i] * e, y = q4[i] * e;
        ka = __builtin_amdgcn_mfma_f32_16x16x4f32(x, x, ka, 0, 0, 0);
        pa = __builtin_amdgcn_mfma_f32_16x16x4f32(y, x, pa, 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 4 * g + i;  // row (token), column m
      if ((r & ~(2 * s - 1)) == (m & ~(2 * s - 1)) && (r & s) && !(m & s)) {
        As[r][m] = beta[r] * ka[i];
        Ps[r][m] = pa[i];
      }
    }
  } else {  // one product each, the key width cut over the waves
    for (int r = wid; r < R; r += 4) {
      const int d = 16 * r + 4 * g;
      const f32x4 k4 = *(const f32x4*)&kx[m][d], q4 = *(const f32x4*)&qx[m][d];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ka = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[i], k4[i], ka, 0, 0, 0);
        pa = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[i], k4[i], pa, 0, 0, 0);
      }
    }
    if (wid) {
      red[wid - 1][0][lane] = ka;
      red[wid - 1][1][lane] = pa;
    }
    __syncthreads();
    if (wid == 0) {
#pragma unroll
      for (int j = 0; j < 3; ++j) {
        ka += red[j][0][lane];
        pa += red[j][1][lane];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 4 * g + i;
        const float e = expf(fminf(Gs[r] - Gs[m], 0.f));
        As[r][m] = r > m ? beta[r] * ka[i] * e : 0.f;
        Ps[r][m] = pa[i] * e;
      }
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // read below by other lanes of this wave
    }
  }
  // Scaled operands: the waves that do not solve for T. Everything they read is in place since the last barrier.
  if constexpr (CHN) __syncthreads();
  if (wid == 0) {
    if (tid < CH) {  // column tid of T, by forward substitution (this wave's own LDS writes, or behind the barrier)
      float x[CH];
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float y = i == tid ? beta[i] : 0.f;
#pragma unroll
        for (int j = 0; j < i; ++j) y = fmaf(-As[i][j], x[j], y);
        x[i] = y;
        ws[L::T + L::sq(i, tid)] = y;
      }
    } else if (tid < 2 * CH) {  // column of P
      const int c = tid - CH;
#pragma unroll
      for (int i = 0; i < CH; ++i) ws[L::P + L::sq(i, c)] = i > c ? Ps[i][c] : (i == c ? dot[i] : 0.f);
    }
    return;
  }
  const int tw = tid - 64;  // 192 threads
  auto gl = [&](int i, int d) { return CHN ? G[i][d] : Gs[i]; };
  for (int e = tw; e < CH * DP / 4; e += 192) {
    const int em = e & 15, d = 16 * (e >> 6) + 4 * (e >> 4 & 3);  // token em, channels d .. d + 3
    const f32x4 k4 = *(const f32x4*)&kx[em][d], q4 = *(const f32x4*)&qx[em][d];
    f32x4 ex;
#pragma unroll
    for (int j = 0; j < 4; ++j) ex[j] = (CHN || j == 0) ? expf(gl(em, d + j)) : ex[0];
    *(f32x4*)(ws + L::KT + 4 * e) = k4 * ex;
    *(f32x4*)(ws + L::QT + 4 * e) = q4 * ex;
  }
  for (int e = tw; e < CH * DP / 4; e += 192) {
    const int d = 16 * (e >> 6) + (e & 15), i = 4 * (e >> 4 & 3);  // channel d, tokens i .. i + 3
    f32x4 y;
#pragma unroll
    for (int j = 0; j < 4; ++j) y[j] = kx[i + j][d] * expf(gl(CH - 1, d) - gl(i + j, d));
    *(f32x4*)(ws + L::KE + 4 * e) = y;
  }
  for (int d = tw; d < DP; d += 192) ws[L::EG + d] = expf(gl(CH - 1, d));
}

// Workgroup = (run, head, 16 value columns); NW waves hold RW 16-row tiles of the state's columns each, as MFMA
// accumulators (row 16 r + 4 g + i, column lane % 16), which are at once the B operands of the products with S0
// (k index of step (r, i): row 16 r + 4 g + i for lane group g). The waves' shares of those products meet in LDS,
// one barrier per chunk; every wave solves for U by itself, and one more finishes the read-outs off the chain from
// chunk to chunk. Operands go straight to registers, two chunks ahead.
// Values stay the 32-bit words they were loaded as until they are used (anything done at the load waits for it); a
// lane's bf16 value is the word's upper half if `odd`
template <typename T> __device__ __forceinline__ float of_word(uint32_t r, bool odd) {
  return __uint_as_float(sizeof(T) == 4 || odd ? (sizeof(T) == 4 ? r : r & 0xffff0000u) : r << 16);
}
template <int RW> struct ScanOps { f32x4 k[RW], q[RW], e[RW], g[RW], t; uint32_t v[4]; };
// uniform base, the lane's byte offset
template <typename V> __device__ __forceinline__ V at(const void* base, uint32_t off) { return *(const V*)((const char*)base + off); }
struct ReadOps { f32x4 t, p; uint32_t v[4]; };

template <typename T, int DP>
__global__ __launch_bounds__(DP / 16 < 4 ? DP * 4 + 64 : 320, DP > 128 ? 2 : 4) void delta_scan_kernel(Args a, Work w, const int* first_chunk) {
  constexpr int R = DP / 16, NW = R < 4 ? R : 4, RW = R / NW;
  using L = Lay<DP>;
  __shared__ f32x4 part[2][NW][2][64];
  const int tid = threadIdx.x, lane = tid & 63, m = lane & 15, g = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int VB = (a.V + 15) / 16, lin = xcd_remap(blockIdx.x, gridDim.x);
  const int vb = lin % VB, h = lin / VB % a.H, ri = lin / (VB * a.H);
  const int4 run = w.runs[ri];
  const int nc = (run.z + CH - 1) / CH, c0 = first_chunk[ri];
  const int col = vb * 16 + m, d0 = 16 * RW * wid;
  const bool ok = col < a.V, live = run.x >= 0 && run.x < a.n_rows;
  float* Sp = a.S + ((long)max(run.x, 0) * a.H + h) * a.D * a.V + (ok ? col : 0);
  const long ldo = (long)a.H * a.V, vc = (long)h * a.V + (ok ? col : 0);
  constexpr int PER = 4 / sizeof(T);  // values per word
  const uint32_t* vp = (const uint32_t*)w.v + (long)run.y * w.ldv / PER;
  const uint32_t ldw = (uint32_t)(w.ldv / PER), vw = (uint32_t)(vc / PER);
  const bool odd = vc & 1;
  float* op = w.o + (long)run.y * ldo;
  const float* wp = w.ws + ((long)h * w.n_chunks + c0) * L::N;
  const uint32_t o_m = 16 * lane, o_s = 16 * (RW * wid * 64 + lane), o_g = 4 * (d0 + 4 * g);  // the wave's row tiles
  auto load_kq = [&](ScanOps<RW>& s, int c) {
    const float* p = wp + (long)min(c, nc - 1) * L::N;
#pragma unroll
    for (int r = 0; r < RW; ++r) {
      s.k[r] = at<f32x4>(p + L::KT + 256 * r, o_s);
      s.q[r] = at<f32x4>(p + L::QT + 256 * r, o_s);
    }
  };
  auto load_tv = [&](auto& s, int c) {  // c < nc
    const uint32_t* p = vp + (long)c * CH * ldw;
    const int last = run.z - 1 - c * CH;
#pragma unroll
    for (int i = 0; i < 4; ++i)  // past the run: beta is 0
      s.v[i] = at<uint32_t>(p, 4 * (__umul24((uint32_t)min(4 * g + i, last), ldw) + vw));
    s.t = at<f32x4>(wp + (long)c * L::N + L::T, o_m);
  };
  auto load_rest = [&](ScanOps<RW>& s, int c) {
    c = min(c, nc - 1);
    load_tv(s, c);
    const float* p = wp + (long)c * L::N;
#pragma unroll
    for (int r = 0; r < RW; ++r) {
      s.e[r] = at<f32x4>(p + L::KE + 256 * r, o_s);
      s.g[r] = at<f32x4>(p + L::EG + 16 * r, o_g);
    }
  };
  // U from the shares of k e^G S0 in buffer b
  auto solve = [&](auto& s, int b) {
#pragma unroll
    for (int i = 0; i < 4; ++i) asm volatile("" : "+v"(s.v[i]));  // nothing of this chunk is used ahead of its barrier
    f32x4 wv = {of_word<T>(s.v[0], odd), of_word<T>(s.v[1], odd), of_word<T>(s.v[2], odd), of_word<T>(s.v[3], odd)}, u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < NW; ++j) wv -= part[b][j][0][lane];
#pragma unroll
    for (int i = 0; i < 4; ++i) u = __builtin_amdgcn_mfma_f32_16x16x4f32(s.t[i], wv[i], u, 0, 0, 0);
    return u;
  };
  if (wid == NW) {  // read-outs
    ReadOps r0, r1;
    auto load = [&](ReadOps& s, int c) {
      c = min(c, nc - 1);
      load_tv(s, c);
      s.p = at<f32x4>(wp + (long)c * L::N + L::P, o_m);
    };
    auto read = [&](ReadOps& s, int c) {
      const int b = c & 1;
      asm volatile("s_barrier" ::: "memory");
      const f32x4 u = solve(s, b);
      f32x4 oo = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < NW; ++j) oo += part[b][j][1][lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) oo = __builtin_amdgcn_mfma_f32_16x16x4f32(s.p[i], u[i], oo, 0, 0, 0);
      float* oc = op + (long)c * CH * ldo;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (ok && 4 * g + i < run.z - c * CH) *(float*)((char*)oc + 4 * (__umul24((uint32_t)(4 * g + i), (uint32_t)ldo) + (uint32_t)vc)) = oo[i];
      load(s, c + 2);
    };
    load(r0, 0);
    load(r1, 1);
    __builtin_amdgcn_s_waitcnt(0x0f70);
    int c = 0;
    for (; c + 1 < nc; c += 2) {
      read(r0, c);
      read(r1, c + 1);
    }
    if (c < nc) read(r0, c);
    return;
  }
  f32x4 S[RW];
  auto chunk = [&](ScanOps<RW>& s, int c) {
    f32x4 x[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}}, o[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int r = 0; r < RW; ++r)
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(s.k[r][i], S[r][i], x[i & 1], 0, 0, 0);
#pragma unroll
    for (int r = 0; r < RW; ++r)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(s.q[r][i], S[r][i], o[i & 1], 0, 0, 0);
    load_kq(s, c + 2);
    const int b = c & 1;
    part[b][wid][0][lane] = x[0] + x[1];
    part[b][wid][1][lane] = o[0] + o[1];
    // the shares are whole; this buffer is written again only behind the next chunk's barrier. Global loads stay in flight
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    asm volatile("s_barrier" ::: "memory");
    const f32x4 u = solve(s, b);
#pragma unroll
    for (int r = 0; r < RW; ++r) {
      asm volatile("" : "+v"(s.g[r]));
      S[r] *= s.g[r];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < RW; ++r) S[r] = __builtin_amdgcn_mfma_f32_16x16x4f32(s.e[r][i], u[i], S[r], 0, 0, 0);
    load_rest(s, c + 2);
  };
  ScanOps<RW> s0, s1;
  load_kq(s0, 0);
  load_rest(s0, 0);
#pragma unroll
  for (int r = 0; r < RW; ++r)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = d0 + 16 * r + 4 * g + i;
      S[r][i] = live && run.w > 0 && ok && d < a.D ? Sp[(long)d * a.V] : 0.f;
    }
  load_kq(s1, 1);
  load_rest(s1, 1);
  __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0): the waits in the loop then count from the loop's own order of loads
  int c = 0;
  for (; c + 1 < nc; c += 2) {
    chunk(s0, c);
    chunk(s1, c + 1);
  }
  if (c < nc) chunk(s0, c);
  if (live && ok) {
#pragma unroll
    for (int r = 0; r < RW; ++r)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = d0 + 16 * r + 4 * g + i;
        if (d < a.D) Sp[(long)d * a.V] = S[r][i];
      }
  }
}

// read-outs -> normed, weighted, gated rows: LPR lanes (a power of two) per (token, head), N columns each at a time
template <typename T, int N>
__global__ __launch_bounds__(256) void delta_out_kernel(Args a, const float* __restrict__ o, long row0, long rows, int LPR) {
  const int lane = threadIdx.x & 63, l = lane & (LPR - 1);
  const long th = row0 + ((long)blockIdx.x * 256 + threadIdx.x) / LPR;  // token * H + head
  const bool in = th < row0 + rows;
  const long t = (in ? th : row0) / a.H;
  const int h = (int)((in ? th : row0) % a.H);
  const float* op = o + (t * a.H + h) * a.V;
  float s = 0.f;
  for (int c = l * N; c < a.V; c += LPR * N) {
    __attribute__((aligned(16))) float ov[N];
    ldf<N>(op + c, ov);
#pragma unroll
    for (int e = 0; e < N; ++e) s = fmaf(ov[e], ov[e], s);
  }
  for (int x = LPR >> 1; x > 0; x >>= 1) s += __shfl_xor(s, x, 64);
  const float r = a.out_scale / sqrtf(s / a.V + a.eps);
  if (!in) return;
  const T* z = (const T*)a.z + t * a.ldz + (long)h * a.V;
  T* out = (T*)a.out + t * a.ldo + (long)h * a.V;
  for (int c = l * N; c < a.V; c += LPR * N) {
    __attribute__((aligned(16))) float ov[N], zv[N], wv[N], y[N];
    ldf<N>(op + c, ov);
    ldn<T, N>(z + c, zv);
    ldn<T, N>((const T*)a.norm_w + c, wv);
#pragma unroll
    for (int e = 0; e < N; ++e) y[e] = ov[e] * r * wv[e] * gate_of(zv[e], a.silu);
    stn<T, N>(out + c, y);
  }
}

// the last projections of every run into its row's ring (behind delta_prep, which reads the old ones)
template <typename T>
__global__ __launch_bounds__(256) void delta_commit_kernel(Args a, const int4* __restrict__ runs) {
  const int4 run = runs[blockIdx.y];
  if (run.x < 0 || run.x >= a.n_rows) return;
  const int C = 2 * a.K * a.D + a.H * a.V;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  T* ring = (T*)a.ring + (long)run.x * a.taps * C;
  const T* x = (const T*)a.x + (long)run.y * a.ldx;
  for (int i = max(0, run.z - a.taps); i < run.z; ++i) ring[(long)((run.w + i) % a.taps) * C + c] = x[(long)i * a.ldx + c];
}

template <typename T, int VEC, int NR>
static int launch_step(const Args& a, int T_, int block, hipStream_t st_) {
  const int ncol = (a.V + VEC - 1) / VEC, RG = block / ncol;
  const size_t lds = (size_t)(3 * a.D + 2 * a.V + 2 * RG * a.V) * 4;
  if (lds > 65536) return -3;
  for (int t0 = 0; t0 < T_; t0 += 65535) {
    Args q = a;
    const long es = sizeof(T);
    q.x = (const char*)a.x + t0 * a.ldx * es; q.b = (const char*)a.b + t0 * a.ldb * es;
    q.a = (const char*)a.a + t0 * a.lda * es; q.z = (const char*)a.z + t0 * a.ldz * es;
    q.out = (char*)a.out + t0 * a.ldo * es; q.row = a.row + t0; q.pos = a.pos + t0;
    dim3 grid(a.H, std::min(T_ - t0, 65535));
    if (block == 256) hipLaunchKernelGGL((delta_step_kernel<T, VEC, NR, 256>), grid, dim3(256), lds, st_, q);
    else if (block == 512) hipLaunchKernelGGL((delta_step_kernel<T, VEC, NR, 512>), grid, dim3(512), lds, st_, q);
    else hipLaunchKernelGGL((delta_step_kernel<T, VEC, NR, 1024>), grid, dim3(1024), lds, st_, q);
    RT_LAUNCH_CHECK();
  }
  return 0;
}

template <typename T>
static int step(const Args& a, int n, hipStream_t st_) {
  const int vec = a.V % 4 == 0 ? 4 : 1, ncol = a.V / vec;
  for (int block = 256; block <= 1024; block *= 2) {
    if (ncol > block) continue;
    const int nr = (a.D + block / ncol - 1) / (block / ncol);
    if (nr > 16 && block < 1024) continue;
    if (vec == 4) {
      if (nr <= 4) return launch_step<T, 4, 4>(a, n, block, st_);
      if (nr <= 8) return launch_step<T, 4, 8>(a, n, block, st_);
      if (nr <= 16) return launch_step<T, 4, 16>(a, n, block, st_);
      return -2;
    }
    if (nr <= 16) return launch_step<T, 1, 16>(a, n, block, st_);
    if (nr <= 64) return launch_step<T, 1, 64>(a, n, block, st_);
    return -2;
  }
  return -2;
}

template <typename T, int DP>
static int runs_(const Args& a, const Work& w, const int* first_chunk, int n_runs, int n_chunks, int t0, int n_tokens,
                 hipStream_t st_) {
  constexpr int N = 16 / sizeof(T);
  auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const bool vec = a.D % N == 0 && a.V % N == 0 && a.ldx % N == 0 && al(a.x) && al(a.ring) && al(a.conv) && al(w.v) &&
                   (!a.channel || (a.lda % N == 0 && al(a.a)));
  const bool vec_out = a.V % N == 0 && a.ldz % N == 0 && a.ldo % N == 0 && al(a.z) && al(a.out) && al(a.norm_w) && al(w.o);
  for (int c0 = 0; c0 < n_chunks; c0 += 65535) {
    Work q = w;
    q.chunks = w.chunks + c0;
    q.chunk0 = c0;
    const dim3 grid(a.H, std::min(n_chunks - c0, 65535));
#define DR_PREP(CHN)                                                                                                          \
  do {                                                                                                                        \
    if (!vec) hipLaunchKernelGGL((delta_prep_kernel<T, DP, CHN, 1, 0>), grid, dim3(256), 0, st_, a, q);                       \
    else if (a.taps == 4) hipLaunchKernelGGL((delta_prep_kernel<T, DP, CHN, N, 4>), grid, dim3(256), 0, st_, a, q);           \
    else hipLaunchKernelGGL((delta_prep_kernel<T, DP, CHN, N, 0>), grid, dim3(256), 0, st_, a, q);                            \
  } while (0)
    if (a.channel) DR_PREP(true);
    else DR_PREP(false);
#undef DR_PREP
    RT_LAUNCH_CHECK();
  }
  hipLaunchKernelGGL((delta_scan_kernel<T, DP>), dim3((unsigned)((long)n_runs * a.H * ((a.V + 15) / 16))),
                     dim3(std::min(DP * 4, 256) + 64), 0, st_, a, w, first_chunk);
  RT_LAUNCH_CHECK();
  int lpr = 1;
  while (lpr < 64 && lpr * (vec_out ? N : 1) < a.V) lpr *= 2;
  const long rows = (long)n_tokens * a.H, row0 = (long)t0 * a.H;
  const dim3 grid((unsigned)((rows * lpr + 255) / 256));
  if (vec_out) hipLaunchKernelGGL((delta_out_kernel<T, N>), grid, dim3(256), 0, st_, a, w.o, row0, rows, lpr);
  else hipLaunchKernelGGL((delta_out_kernel<T, 1>), grid, dim3(256), 0, st_, a, w.o, row0, rows, lpr);
  RT_LAUNCH_CHECK();
  const int C = 2 * a.K * a.D + a.H * a.V;
  hipLaunchKernelGGL((delta_commit_kernel<T>), dim3((C + 255) / 256, n_runs), dim3(256), 0, st_, a, w.runs);
  RT_LAUNCH_CHECK();
  return 0;
}

static int pad_d(int D) { return D <= 32 ? 32 : (D <= 64 ? 64 : (D <= 128 ? 128 : (D <= 256 ? 256 : 0))); }

}  // namespace dr
}  // namespace rt

using namespace rt;
using namespace rt::dr;

struct RtDelta {  // mirrors csrc/host/bind_layered.cpp
  const void* x; long ldx; const void* b; long ldb; const void* a; long lda; const void* z; long ldz;
  const void* conv; const float* A_log; const float* dt; const void* norm_w; float eps;
  const int* row; const int* pos; float* S; void* ring; int n_rows; void* out; long ldo; float out_scale;
  int H, K, D, V, taps, channel, silu;
};

static Args make_args(const RtDelta& d) {
  return Args{d.x, d.ldx, d.b, d.ldb, d.a, d.lda, d.z, d.ldz, d.conv, d.A_log, d.dt, d.norm_w, d.eps, d.row, d.pos, d.S,
              d.ring, d.n_rows, d.out, d.ldo, d.out_scale, d.H, d.K, d.D, d.V, d.taps, d.channel, d.silu};
}

// tokens [0, n): one per request
extern "C" int rt_delta_step(int f32, const RtDelta* d, int n, hipStream_t stream) {
  if (n <= 0) return 0;
  const Args a = make_args(*d);
  return f32 ? step<float>(a, n, stream) : step<bf16_t>(a, n, stream);
}

// floats of workspace per (chunk, head); 0: the key width is not supported
extern "C" long rt_delta_ws(int D) {
  const int dp = pad_d(D);
  return dp ? 3L * CH * dp + dp + 2 * CH * CH : 0;
}

// runs of several tokens: tokens [t0, t0 + n_tokens) of the batch, n_chunks chunks in all
extern "C" int rt_delta_runs(int f32, const RtDelta* d, const void* runs, const void* chunks, const int* first_chunk,
                             int n_runs, int n_chunks, int t0, int n_tokens, float* ws, void* v, float* o,
                             hipStream_t stream) {
  if (n_runs <= 0) return 0;
  if (n_runs > 65535) return -1;
  const Args a = make_args(*d);
  const Work w{(const int4*)runs, (const int2*)chunks, ws, n_chunks, 0, ((long)a.H * a.V + 1) / 2 * 2, v, o};
#define DR_(DP)                                                                                       \
  return f32 ? runs_<float, DP>(a, w, first_chunk, n_runs, n_chunks, t0, n_tokens, stream)            \
             : runs_<bf16_t, DP>(a, w, first_chunk, n_runs, n_chunks, t0, n_tokens, stream)
  switch (pad_d(a.D)) {
    case 32: DR_(32);
    case 64: DR_(64);
    case 128: DR_(128);
    case 256: DR_(256);
  }
#undef DR_
  return -2;
}
