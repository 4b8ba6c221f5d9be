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
//   portions:     delta_prep (chunks of 16 tokens, all in parallel) -> delta_scan (chunks in order, fp32 MFMA)
//                 -> delta_out (norm, gate), delta_commit (ring)
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

__device__ __forceinline__ float sigmoid(float x) { return 1.f / (1.f + expf(-x)); }
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
// one token per request. Thread = VEC value columns x NR key rows of the state, held in registers; the
// projections' part (convolutions, unit norms, decays) runs while the state is on its way.
// ---------------------------------------------------------------------------------------------
template <typename T, int VEC, int NR, int BLOCK>
__global__ __launch_bounds__(BLOCK) void delta_step_kernel(Args a) {
  extern __shared__ float sm[];  // k, q (unit, decayed later), g [D]; v, o [V]; sums [2][RG][V]; red [2 * BLOCK / 64]
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int D = a.D, V = a.V, kh = h / (a.H / a.K);
  const int ncol = (V + VEC - 1) / VEC, RG = BLOCK / ncol;
  float* ks = sm;
  float* qs = ks + D;
  float* gs = qs + D;
  float* vs = gs + D;
  float* os = vs + V;
  float* sum = os + V;
  const int row = a.row[t], pos = max(a.pos[t], 0);
  const bool live = row >= 0 && row < a.n_rows, carry = live && pos > 0;
  const int cg = tid % ncol, rg = tid / ncol;
  const bool mine = rg < RG;
  float* Sp = a.S + (((long)max(row, 0) * a.H + h) * D) * V + cg * VEC;
  float s[NR][VEC];
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    const int d = rg + j * RG;
#pragma unroll
    for (int e = 0; e < VEC; ++e) s[j][e] = 0.f;
    if (carry && mine && d < D) {
      if constexpr (VEC == 4) {
        const float4 v = *(const float4*)(Sp + (long)d * V);
        s[j][0] = v.x; s[j][1] = v.y; s[j][2] = v.z; s[j][3] = v.w;
      } else {
        s[j][0] = Sp[(long)d * V];
      }
    }
  }
  const int KD = a.K * D, C = 2 * KD + a.H * V;
  const T* xt = (const T*)a.x + (long)t * a.ldx;
  T* ring = (T*)a.ring + (long)max(row, 0) * a.taps * C;
  const Conv<T> conv{a, xt, carry ? ring : nullptr, pos, C};
  for (int i = tid; i < 2 * D + V; i += BLOCK) {
    const int c = i < D ? kh * D + i : (i < 2 * D ? KD + kh * D + i - D : 2 * KD + h * V + i - 2 * D);
    const float y = conv(pos, c);
    (i < D ? qs[i] : (i < 2 * D ? ks[i - D] : vs[i - 2 * D])) = y;
    // the slot of this position is read by nobody at this position; heads that share a key head share the write
    if (live && (i >= 2 * D || h % (a.H / a.K) == 0)) ring[(long)(pos % a.taps) * C + c] = xt[c];
  }
  const float A = expf(a.A_log[h]);
  if (a.channel) {
    for (int d = tid; d < D; d += BLOCK)
      gs[d] = expf(-A * softplus(ld((const T*)a.a + (long)t * a.lda + (long)h * D + d) + a.dt[(long)h * D + d]));
  } else {
    const float g = expf(-A * softplus(ld((const T*)a.a + (long)t * a.lda + h) + a.dt[h]));
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
  const float beta = sigmoid(ld((const T*)a.b + (long)t * a.ldb + h));
  float pk[VEC], pq[VEC];
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
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      sum[rg * V + cg * VEC + e] = pk[e];
      sum[(RG + rg) * V + cg * VEC + e] = pq[e];
    }
  }
  __syncthreads();
  float u[VEC];
  if (mine) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const int c = cg * VEC + e;
      float sk = 0.f, sq = 0.f;
      for (int r = 0; r < RG; ++r) {
        sk += sum[r * V + c];
        sq += sum[(RG + r) * V + c];
      }
      u[e] = beta * (vs[c] - sk);
      if (rg == 0) os[c] = fmaf(qk, u[e], sq);  // S^T q behind the write
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
  for (int c = tid; c < V; c += BLOCK)
    st((T*)a.out + (long)t * a.ldo + (long)h * V + c,
       os[c] * r * ld((const T*)a.norm_w + c) * gate_of(ld((const T*)a.z + (long)t * a.ldz + (long)h * V + c), a.silu));
}

// ---------------------------------------------------------------------------------------------
// portions
// ---------------------------------------------------------------------------------------------
// runs: {row, first token, tokens, position of the first}; chunks: {run, chunk of the run}, a run's chunks
// consecutive. Workspace per (chunk, head): KT, QT, KE [CH][DP], EG [DP], T, P [CH][CH] floats.
struct Work {
  const int4* runs; const int2* chunks;
  float* ws;
  void* v;      // [N, H * V] convolved values, rows of the batch's tokens
  float* o;     // [N, H * V] read-outs
};
template <int DP> struct Lay {
  static constexpr int KT = 0, QT = CH * DP, KE = 2 * CH * DP, EG = 3 * CH * DP, T = EG + DP, P = T + CH * CH, N = P + CH * CH;
};

template <typename T, int DP>
__global__ __launch_bounds__(256) void delta_prep_kernel(Args a, Work w) {
  constexpr int LD = DP + 4, R = DP / 16;
  using L = Lay<DP>;
  __shared__ __attribute__((aligned(16))) float kx[CH][LD], qx[CH][LD], G[CH][LD];
  __shared__ float As[CH][CH + 1], Ps[CH][CH + 1], beta[CH], dot[CH];
  const int h = blockIdx.x, ci = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int2 ck = w.chunks[ci];
  const int4 run = w.runs[ck.x];
  const int n = min(CH, run.z - ck.y * CH), p0 = run.w + ck.y * CH, t0 = run.y + ck.y * CH;
  const int D = a.D, V = a.V, kh = h / (a.H / a.K), KD = a.K * D, C = 2 * KD + a.H * V;
  const bool carry = run.x >= 0 && run.x < a.n_rows && run.w > 0;
  const Conv<T> conv{a, (const T*)a.x + (long)run.y * a.ldx,
                     carry ? (const T*)a.ring + (long)run.x * a.taps * C : nullptr, run.w, C};
  const float A = expf(a.A_log[h]);
  if (tid < CH) beta[tid] = tid < n ? sigmoid(ld((const T*)a.b + (long)(t0 + tid) * a.ldb + h)) : 0.f;
  for (int e = tid; e < CH * DP; e += 256) {
    const int i = e / DP, d = e % DP;
    float k = 0.f, q = 0.f, g = 0.f;
    if (i < n && d < D) {
      q = conv(p0 + i, kh * D + d);
      k = conv(p0 + i, KD + kh * D + d);
      g = a.channel ? -A * softplus(ld((const T*)a.a + (long)(t0 + i) * a.lda + (long)h * D + d) + a.dt[(long)h * D + d])
                    : -A * softplus(ld((const T*)a.a + (long)(t0 + i) * a.lda + h) + a.dt[h]);
    }
    kx[i][d] = k;
    qx[i][d] = q;
    G[i][d] = g;
  }
  for (int e = tid; e < n * V; e += 256) {
    const int i = e / V, c = e % V;
    st((T*)w.v + (long)(t0 + i) * a.H * V + (long)h * V + c, conv(p0 + i, 2 * KD + h * V + c));
  }
  __syncthreads();
  for (int i = wid; i < CH; i += 4) {  // unit vectors
    float kk = 0.f, qq = 0.f, qk = 0.f;
    for (int d = lane; d < D; d += 64) {
      kk += kx[i][d] * kx[i][d];
      qq += qx[i][d] * qx[i][d];
      qk += qx[i][d] * kx[i][d];
    }
    const float ik = 1.f / sqrtf(wave_sum(kk) + 1e-6f), iq = 1.f / sqrtf(wave_sum(qq) + 1e-6f) / sqrtf((float)D);
    qk = wave_sum(qk);
    for (int d = lane; d < D; d += 64) {
      kx[i][d] *= ik;
      qx[i][d] *= iq;
    }
    if (lane == 0) dot[i] = qk * ik * iq;
  }
  for (int d = tid; d < DP; d += 256) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      s += G[i][d];
      G[i][d] = s;
    }
  }
  __syncthreads();
  {  // A and P: wave = level of the split, half size s
    const int m = lane & 15, g = lane >> 4, s = 8 >> wid;
    const int piv = (m & ~(2 * s - 1)) + s - 1;
    f32x4 ka = {0.f, 0.f, 0.f, 0.f}, pa = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int r = 0; r < R; ++r) {
      const int d = 16 * r + 4 * g;
      const float4 k4 = *(const float4*)&kx[m][d], q4 = *(const float4*)&qx[m][d];
      const float4 g4 = *(const float4*)&G[m][d], v4 = *(const float4*)&G[piv][d];
      const float kk[4] = {k4.x, k4.y, k4.z, k4.w}, qq[4] = {q4.x, q4.y, q4.z, q4.w};
      const float dd[4] = {g4.x - v4.x, g4.y - v4.y, g4.z - v4.z, g4.w - v4.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float e = expf(-fabsf(dd[i]));
        const float x = kk[i] * e, y = qq[i] * e;
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
  }
  __syncthreads();
  float* ws = w.ws + ((long)ci * a.H + h) * L::N;
  if (tid < CH) {  // column tid of T, by forward substitution
    float x[CH];
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      float y = i == tid ? beta[i] : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) y = fmaf(-As[i][j], x[j], y);
      x[i] = y;
      ws[L::T + i * CH + tid] = y;
    }
  }
  if (tid >= 64 && tid < 64 + CH) {  // column of P
    const int c = tid - 64;
#pragma unroll
    for (int i = 0; i < CH; ++i) ws[L::P + i * CH + c] = i > c ? Ps[i][c] : (i == c ? dot[i] : 0.f);
  }
  for (int e = tid; e < CH * DP / 4; e += 256) {
    const int i = e / (DP / 4), d = e % (DP / 4) * 4;
    const float4 k4 = *(const float4*)&kx[i][d], q4 = *(const float4*)&qx[i][d];
    const float4 g4 = *(const float4*)&G[i][d], l4 = *(const float4*)&G[CH - 1][d];
    const float ex = expf(g4.x), ey = expf(g4.y), ez = expf(g4.z), ew = expf(g4.w);
    *(float4*)(ws + L::KT + i * DP + d) = make_float4(k4.x * ex, k4.y * ey, k4.z * ez, k4.w * ew);
    *(float4*)(ws + L::QT + i * DP + d) = make_float4(q4.x * ex, q4.y * ey, q4.z * ez, q4.w * ew);
    *(float4*)(ws + L::KE + i * DP + d) = make_float4(k4.x * expf(l4.x - g4.x), k4.y * expf(l4.y - g4.y),
                                                      k4.z * expf(l4.z - g4.z), k4.w * expf(l4.w - g4.w));
  }
  for (int d = tid; d < DP; d += 256) ws[L::EG + d] = expf(G[CH - 1][d]);
}

// Workgroup = (run, head, 64 value columns), wave = 16 columns: the state's columns as DP / 16 MFMA
// accumulators (row 16 r + 4 g + i, column lane % 16), which are at once the B operands of the products with
// S0 (k index of step (r, i): row 16 r + 4 g + i for lane group g). The chunk's operands are shared through
// LDS, two buffers, the next chunk's loads in flight during the products.
template <typename T, int DP>
__global__ __launch_bounds__(256) void delta_scan_kernel(Args a, Work w, const int* first_chunk) {
  constexpr int LD = DP + 4, R = DP / 16;
  using L = Lay<DP>;
  constexpr int N4 = L::N / 4, NLD = (N4 + 255) / 256;
  // LDS image of a chunk: KT, QT, KE rows padded to LD, then EG, T, P
  constexpr int IK = 0, IQ = CH * LD, IE = 2 * CH * LD, IG = 3 * CH * LD, IT = IG + DP, IP = IT + CH * CH, IN = IP + CH * CH;
  __shared__ __attribute__((aligned(16))) float sm[2][IN];
  const int tid = threadIdx.x, lane = tid & 63, m = lane & 15, g = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int VB = (a.V + 63) / 64;
  const int vb = blockIdx.x % VB, h = blockIdx.x / VB % a.H, ri = blockIdx.x / (VB * a.H);
  const int4 run = w.runs[ri];
  const int nc = (run.z + CH - 1) / CH, c0 = first_chunk[ri];
  const int col = vb * 64 + wid * 16 + m;
  const bool ok = col < a.V;
  const bool live = run.x >= 0 && run.x < a.n_rows;
  float* Sp = a.S + ((long)max(run.x, 0) * a.H + h) * a.D * a.V + (ok ? col : 0);
  f32x4 S[R];
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * r + 4 * g + i;
      S[r][i] = live && run.w > 0 && ok && d < a.D ? Sp[(long)d * a.V] : 0.f;
    }
  float4 pre[NLD];
  auto load = [&](int c) {
    const float4* src = (const float4*)(w.ws + ((long)(c0 + c) * a.H + h) * L::N);
#pragma unroll
    for (int j = 0; j < NLD; ++j) pre[j] = src[min(tid + 256 * j, N4 - 1)];
  };
  auto place = [&](int b) {
#pragma unroll
    for (int j = 0; j < NLD; ++j) {
      const int e = (tid + 256 * j) * 4;
      if (e >= L::N) continue;
      const int at = e < L::EG ? e / DP * LD + e % DP : IG + e - L::EG;
      *(float4*)&sm[b][at] = pre[j];
    }
  };
  const long ldv = (long)a.H * a.V;
  const T* vp = (const T*)w.v + (long)run.y * ldv + (long)h * a.V + (ok ? col : 0);
  float* op = w.o + (long)run.y * ldv + (long)h * a.V + (ok ? col : 0);
  float vn[4];
  auto load_v = [&](int c) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = c * CH + 4 * g + i;
      vn[i] = ok && t < run.z ? ld(vp + (long)t * ldv) : 0.f;
    }
  };
  load(0);
  load_v(0);
  for (int c = 0; c < nc; ++c) {
    const float* s = sm[c & 1];
    place(c & 1);
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = vn[i];
    __syncthreads();  // this image is whole; the other one is written only after the next barrier's arrivals
    if (c + 1 < nc) {
      load(c + 1);
      load_v(c + 1);
    }
    f32x4 x[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}}, o[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const f32x4 k4 = *(const f32x4*)(s + IK + m * LD + 16 * r + 4 * g), q4 = *(const f32x4*)(s + IQ + m * LD + 16 * r + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        x[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[i], S[r][i], x[i & 1], 0, 0, 0);
        o[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[i], S[r][i], o[i & 1], 0, 0, 0);
      }
    }
    f32x4 wv, u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) wv[i] = v[i] - (x[0][i] + x[1][i]);
    const f32x4 t4 = *(const f32x4*)(s + IT + m * CH + 4 * g), p4 = *(const f32x4*)(s + IP + m * CH + 4 * g);
#pragma unroll
    for (int i = 0; i < 4; ++i) u = __builtin_amdgcn_mfma_f32_16x16x4f32(t4[i], wv[i], u, 0, 0, 0);
    f32x4 oo = o[0] + o[1];
#pragma unroll
    for (int i = 0; i < 4; ++i) oo = __builtin_amdgcn_mfma_f32_16x16x4f32(p4[i], u[i], oo, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      f32x4 d = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 4; ++i)
        d = __builtin_amdgcn_mfma_f32_16x16x4f32(s[IE + (4 * g + i) * LD + 16 * r + m], u[i], d, 0, 0, 0);
      const f32x4 eg = *(const f32x4*)(s + IG + 16 * r + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) S[r][i] = fmaf(S[r][i], eg[i], d[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = c * CH + 4 * g + i;
      if (ok && t < run.z) op[(long)t * ldv] = oo[i];
    }
  }
  if (live && ok) {
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * r + 4 * g + i;
        if (d < a.D) Sp[(long)d * a.V] = S[r][i];
      }
  }
}

// read-outs -> normed, weighted, gated rows: wave = one (token, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(Args a, const float* __restrict__ o, int t0) {
  const int lane = threadIdx.x & 63, h = blockIdx.x * 4 + (threadIdx.x >> 6);
  const long t = t0 + (long)blockIdx.y;
  if (h >= a.H) return;
  const float* op = o + (t * a.H + h) * a.V;
  float s = 0.f;
  for (int c = lane; c < a.V; c += 64) s += op[c] * op[c];
  const float r = a.out_scale / sqrtf(wave_sum(s) / a.V + a.eps);
  for (int c = lane; c < a.V; c += 64)
    st((T*)a.out + t * a.ldo + (long)h * a.V + c,
       op[c] * r * ld((const T*)a.norm_w + c) * gate_of(ld((const T*)a.z + t * a.ldz + (long)h * a.V + c), a.silu));
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
  for (int c0 = 0; c0 < n_chunks; c0 += 65535) {
    Work q = w;
    q.chunks = w.chunks + c0;
    q.ws = w.ws + (long)c0 * a.H * Lay<DP>::N;
    hipLaunchKernelGGL((delta_prep_kernel<T, DP>), dim3(a.H, std::min(n_chunks - c0, 65535)), dim3(256), 0, st_, a, q);
    RT_LAUNCH_CHECK();
  }
  hipLaunchKernelGGL((delta_scan_kernel<T, DP>), dim3((unsigned)((long)n_runs * a.H * ((a.V + 63) / 64))), dim3(256), 0, st_, a,
                     w, first_chunk);
  RT_LAUNCH_CHECK();
  for (int c = 0; c < n_tokens; c += 65535) {
    hipLaunchKernelGGL((delta_out_kernel<T>), dim3((a.H + 3) / 4, std::min(n_tokens - c, 65535)), dim3(256), 0, st_, a, w.o, t0 + c);
    RT_LAUNCH_CHECK();
  }
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
  const Work w{(const int4*)runs, (const int2*)chunks, ws, v, o};
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
