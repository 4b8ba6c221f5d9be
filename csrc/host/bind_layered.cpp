// Python bindings of the kernels behind layered decoders (latent attention over a paged cache, mixture
// of experts, branch norms, shape-free GEMM): checked wrappers on the current HIP stream. Index tensors
// (page table, rows, positions, expert offsets) are bounded inside the kernels; everything a kernel's
// grid or strides assume is checked here.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime_api.h>

#include <mutex>
#include <unordered_map>
#include <vector>

extern "C" {
int rt_branch_norm(int, int, float*, const void*, long, int, const void*, const void*, const void*, float, void*,
                   const void*, const long*, int, const float*, const int*, int, int, int, float, hipStream_t);
int rt_gemm_any(int, int, const void*, long, long, const void*, long, long, void*, long, long, int, int, int, int,
                const int*, const int*, hipStream_t);
int rt_glu_any(int, const void*, long, void*, long, int, const float*, hipStream_t);
int rt_act_any(int, const float*, void*, long, int, hipStream_t);
int rt_gate_mul(int, void*, const void*, long, long, int, hipStream_t);
int rt_moe_route(const float*, long, int, long, const float*, int, int, int, int, int, int*, float*, hipStream_t);
int rt_moe_sort(const int*, int, int, int, int*, int*, int*, int, int, void*, int*, hipStream_t);
int rt_moe_rows(const void*, long, const int*, const void*, long, long, void*, long, const int*, int, int, int, int, int,
                int, int, const float*, hipStream_t);
int rt_gemm_grouped(const void*, long, const int*, const void*, long, long, void*, long, const void*, const int*, int,
                    int, int, int, const float*, const void*, int, hipStream_t);
int rt_latent_prep(int, void*, long, int, const void*, float, const float*, const float*, int, int, const int*,
                   const int*, void*, const int*, int, int, int, void*, int, int, int, int, int, int, hipStream_t);
int rt_head_gemm(const void*, long, long, const void*, long, long, void*, long, long, int, int, int, int, const void*,
                 long, hipStream_t);
int rt_latent_decode_ok(int, int);
int rt_latent_decode(const void*, const void*, const int*, int, int, int, const int*, const int*, float*, float*, int,
                     int, int, int, int, float, hipStream_t);
int rt_partition_merge(const float*, const float*, const float*, void*, long, int, int, int, int, float, hipStream_t);
int rt_latent_gather(int, const void*, const int*, int, int, const void*, int, int, void*, int, hipStream_t);
int rt_latent_prefill_ok(int, int, int);
int rt_latent_prefill(const void*, long, const void*, long, int, int, const float*, const void*, long, void*, long,
                      const void*, const void*, int, int, int, int, int, float, hipStream_t);
int rt_window_prep(int, void*, long, int, int, int, const void*, const void*, float, const float*, const float*, int, int,
                   const int*, const int*, void*, const int*, int, int, int, int, int, int, int, int, hipStream_t);
int rt_window_decode_ok(int, int, int, int);
int rt_window_decode(const void*, long, const void*, const int*, int, int, int, const int*, const int*, float*, float*, int,
                     int, int, int, int, int, int, int, float, float, hipStream_t);
int rt_window_prefill_ok(int, int);
int rt_window_prefill(const void*, long, const void*, const int*, int, int, int, void*, long, const void*, const void*, int,
                      int, int, int, int, int, int, float, float, float, hipStream_t);
int rt_window_any(int, const void*, long, const void*, const int*, int, int, int, const int*, const int*, void*, long, int,
                  int, int, int, int, int, int, float, float, float, hipStream_t);
struct RtDelta {  // mirrors csrc/kernels/delta_rule.hip
  const void* x; long ldx; const void* b; long ldb; const void* a; long lda; const void* z; long ldz;
  const void* conv; const float* A_log; const float* dt; const void* norm_w; float eps;
  const int* row; const int* pos; float* S; void* ring; int n_rows; void* out; long ldo; float out_scale;
  int H, K, D, V, taps, channel, silu;
};
int rt_delta_step(int, const RtDelta*, int, hipStream_t);
long rt_delta_ws(int);
int rt_delta_runs(int, const RtDelta*, const void*, const void*, const int*, int, int, int, int, float*, void*, float*,
                  hipStream_t);
int rt_latent_any(int, const void*, const void*, const int*, int, int, int, const int*, const int*, const float*, void*,
                  int, int, int, int, float, hipStream_t);
}

namespace py = pybind11;

namespace {

using at::Tensor;
using c10::optional;

hipStream_t stream() { return c10::hip::getCurrentHIPStream().stream(); }
void rc_ok(int rc, const char* what) { TORCH_CHECK(rc == 0, what, " launch failed (code ", rc, ")"); }
bool is_f32(const Tensor& t) { return t.scalar_type() == at::kFloat; }
bool has(const optional<Tensor>& t) { return t.has_value() && t->defined(); }
void* ptr(const optional<Tensor>& t) { return has(t) ? t->data_ptr() : nullptr; }
void act_type(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda() && (t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat), n,
              ": GPU tensor of bf16 or fp32 expected");
}
void same(const Tensor& a, const Tensor& b, const char* n) {
  TORCH_CHECK(a.scalar_type() == b.scalar_type() && b.is_cuda(), n, ": operand types differ");
}
void ints(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous(), n, ": contiguous int32 GPU tensor expected");
}
void f32c(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda() && is_f32(t) && t.is_contiguous(), n, ": contiguous fp32 GPU tensor expected");
}
void rows(const Tensor& t, const char* n) {
  TORCH_CHECK(t.dim() == 2 && (t.stride(1) == 1 || t.size(1) == 1), n, ": 2-D rows expected");
}
bool al16(const Tensor& t) { return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0; }
struct Glu {
  float v[3];
  explicit Glu(const std::vector<double>& g) {
    TORCH_CHECK(g.size() == 3, "glu: {limit, alpha, offset} expected");
    for (int i = 0; i < 3; ++i) v[i] = (float)g[i];
  }
};
const Tensor& zero_page(const Tensor& like) {
  static std::mutex mu;
  static auto* map = new std::unordered_map<int, Tensor>();
  std::lock_guard<std::mutex> g(mu);
  auto it = map->find(like.get_device());
  if (it == map->end())
    it = map->emplace(like.get_device(), at::zeros({2048}, like.options().dtype(at::kBFloat16))).first;
  return it->second;
}

// x [T, H] fp32 in place; kind 0 none / embedding, 1 rows of the activation type, 2 fp32 slabs
// [nsplit, T, H], 3 pairs (activation type), 4 pairs (fp32). Returns h (plain: x rounded, without w_next) or
// None.
py::object branch_norm(Tensor x, int64_t kind, const optional<Tensor>& y, int64_t nsplit, const optional<Tensor>& w_branch,
                       const optional<Tensor>& w_next, const optional<Tensor>& table, const optional<Tensor>& ids,
                       const optional<Tensor>& pair_w, const optional<Tensor>& pair_pos, double eps,
                       const optional<Tensor>& scale, double next_mul, bool plain) {
  f32c(x, "branch_norm x");
  TORCH_CHECK(x.dim() == 2, "branch_norm: x [T, H]");
  const int64_t T = x.size(0), H = x.size(1);
  TORCH_CHECK(kind >= 0 && kind <= 4 && (kind == 0 || has(w_branch)) && (kind != 0 || !has(w_branch) || has(table)) &&
                  !(plain && has(w_next)), "branch_norm: kind / w_branch");
  const Tensor& like = has(w_branch) ? *w_branch : (has(w_next) ? *w_next : *table);
  act_type(like, "branch_norm weights");
  for (const auto* w : {&w_branch, &w_next, &scale})
    if (has(*w)) TORCH_CHECK((*w)->numel() == H && (*w)->is_contiguous() && (*w)->scalar_type() == like.scalar_type(), "branch_norm: weights");
  int64_t K = 0, vocab = 0;
  if (kind == 0) {
    if (has(table)) {
      TORCH_CHECK(table->dim() == 2 && table->size(1) == H && table->is_contiguous() && has(ids) && ids->is_cuda() &&
                      ids->scalar_type() == at::kLong && ids->is_contiguous() && ids->numel() == T,
                  "branch_norm: table / ids");
      same(like, *table, "branch_norm table");
      vocab = table->size(0);
    }
  } else {
    TORCH_CHECK(has(y) && y->is_contiguous() && y->is_cuda(), "branch_norm: y");
    if (kind == 2) {
      TORCH_CHECK(is_f32(*y) && nsplit >= 1 && y->numel() >= nsplit * T * H, "branch_norm: slabs");
    } else if (kind == 1) {
      same(like, *y, "branch_norm y");
      TORCH_CHECK(y->numel() == T * H, "branch_norm: y [T, H]");
    } else {
      TORCH_CHECK(y->dim() == 2 && y->size(1) == H && has(pair_w) && has(pair_pos), "branch_norm: pairs");
      TORCH_CHECK(kind == 4 ? is_f32(*y) : y->scalar_type() == like.scalar_type(), "branch_norm: pair type");
      f32c(*pair_w, "branch_norm pair_w");
      ints(*pair_pos, "branch_norm pair_pos");
      TORCH_CHECK(pair_w->dim() == 2 && pair_w->size(0) == T && pair_pos->numel() == pair_w->numel() &&
                      y->size(0) == pair_w->numel(),
                  "branch_norm: one row of y per pair");
      K = pair_w->size(1);
    }
  }
  Tensor h;
  const bool want = has(w_next) || plain;
  if (want) h = at::empty({T, H}, like.options());
  rc_ok(rt_branch_norm(is_f32(like), (int)kind, x.data_ptr<float>(), ptr(y), T * H, (int)nsplit, ptr(w_branch), ptr(scale),
                       ptr(w_next), (float)next_mul, want ? h.data_ptr() : nullptr, ptr(table), (const long*)ptr(ids),
                       (int)vocab, (const float*)ptr(pair_w), (const int*)ptr(pair_pos), (int)K, (int)T, (int)H, (float)eps, stream()),
        "branch_norm");
  return want ? py::cast(h) : py::none();
}

// out = a w^T. 2-D operands; 3-D: batched (strided views with unit last stride); offs: grouped (w 3-D,
// a / out 2-D rows sorted by group, row_map optional)
Tensor gemm_any(const Tensor& a, const Tensor& w, bool out_f32, optional<Tensor> out, const optional<Tensor>& offs,
                const optional<Tensor>& row_map) {
  act_type(a, "gemm_any a");
  same(a, w, "gemm_any");
  const bool grouped = has(offs);
  const bool batched = a.dim() == 3;
  const int64_t B = (batched || grouped) ? w.size(0) : 1;
  TORCH_CHECK(w.dim() == ((batched || grouped) ? 3 : 2) && (batched || a.dim() == 2) && !(batched && grouped), "gemm_any: dims");
  TORCH_CHECK(!batched || a.size(0) == B, "gemm_any: batch");
  const int64_t K = a.size(-1), N = w.size(-2);
  int64_t M = a.size(-2);
  TORCH_CHECK(w.size(-1) == K && (a.stride(-1) == 1 || K == 1) && (w.stride(-1) == 1 || K == 1), "gemm_any: K / strides");
  if (grouped) {
    ints(*offs, "gemm_any offs");
    TORCH_CHECK(offs->numel() == B + 1, "gemm_any: offs [groups + 1]");
    if (has(row_map)) {
      ints(*row_map, "gemm_any row_map");
      M = row_map->numel();
    }
  }
  const auto odt = (out_f32 || is_f32(a)) ? at::kFloat : at::kBFloat16;
  Tensor c;
  if (has(out)) {
    c = *out;
    TORCH_CHECK(c.scalar_type() == odt && c.size(-1) == N && c.size(-2) == M && (c.stride(-1) == 1 || N == 1) &&
                    c.dim() == (batched ? 3 : 2) && (!batched || c.size(0) == B), "gemm_any: out");
  } else {
    c = batched ? at::empty({B, M, N}, a.options().dtype(odt)) : at::empty({M, N}, a.options().dtype(odt));
  }
  rc_ok(rt_gemm_any(is_f32(a), out_f32, a.data_ptr(), a.stride(-2), batched ? a.stride(0) : 0, w.data_ptr(), w.stride(-2),
                    w.dim() == 3 ? w.stride(0) : 0, c.data_ptr(), c.stride(-2), batched ? c.stride(0) : 0, (int)M, (int)N,
                    (int)K, (int)B, (const int*)ptr(offs), (const int*)ptr(row_map), stream()),
        "gemm_any");
  return c;
}

// out[b] = a[b] w[b]^T at few rows (bf16; strided 3-D views), times sigmoid(gate [rows, batch * N])
void head_gemm(const Tensor& a, const Tensor& w, Tensor out, const optional<Tensor>& gate) {
  TORCH_CHECK(a.is_cuda() && w.is_cuda() && a.scalar_type() == at::kBFloat16 && w.scalar_type() == at::kBFloat16 &&
                  out.scalar_type() == at::kBFloat16, "head_gemm: bf16");
  TORCH_CHECK(a.dim() == 3 && w.dim() == 3 && out.dim() == 3 && a.size(0) == w.size(0) && out.size(0) == w.size(0) &&
                  a.size(2) == w.size(2) && out.size(1) == a.size(1) && out.size(2) == w.size(1) && a.stride(2) == 1 &&
                  w.stride(2) == 1 && out.stride(2) == 1 && al16(a) && al16(w), "head_gemm: shapes");
  if (has(gate)) {
    rows(*gate, "head_gemm gate");
    TORCH_CHECK(gate->is_cuda() && gate->scalar_type() == at::kBFloat16 && gate->size(0) >= a.size(1) &&
                    gate->size(1) == w.size(0) * w.size(1), "head_gemm: gate");
  }
  rc_ok(rt_head_gemm(a.data_ptr(), a.stride(1), a.stride(0), w.data_ptr(), w.stride(1), w.stride(0), out.data_ptr(),
                     out.stride(1), out.stride(0), (int)a.size(1), (int)w.size(1), (int)w.size(2), (int)w.size(0), ptr(gate),
                     has(gate) ? gate->stride(0) : 0, stream()),
        "head_gemm");
}

Tensor glu_any(const Tensor& gu, const std::vector<double>& glu) {
  act_type(gu, "glu_any");
  rows(gu, "glu_any");
  TORCH_CHECK(gu.size(1) % 2 == 0, "glu_any: [T, 2F]");
  Tensor y = at::empty({gu.size(0), gu.size(1) / 2}, gu.options());
  rc_ok(rt_glu_any(is_f32(gu), gu.data_ptr(), gu.stride(0), y.data_ptr(), gu.size(0), (int)(gu.size(1) / 2), Glu(glu).v, stream()),
        "glu_any");
  return y;
}

// activation of an fp32 product: act 8 = max(x, 0)^2
Tensor act_any(const Tensor& x, int64_t act, bool out_f32) {
  f32c(x, "act_any");
  Tensor y = at::empty(x.sizes(), x.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  rc_ok(rt_act_any(out_f32, x.data_ptr<float>(), y.data_ptr(), x.numel(), (int)act, stream()), "act_any");
  return y;
}

void gate_mul(Tensor a, const Tensor& g) {
  act_type(a, "gate_mul");
  same(a, g, "gate_mul");
  rows(g, "gate_mul");
  TORCH_CHECK(a.is_contiguous() && a.dim() == 2 && g.size(0) == a.size(0) && g.size(1) == a.size(1), "gate_mul: shapes");
  rc_ok(rt_gate_mul(is_f32(a), a.data_ptr(), g.data_ptr(), g.stride(0), a.size(0), (int)a.size(1), stream()), "gate_mul");
}

// logits [T, >= E] fp32, or [nslab * T, ..] split-K slabs -> (idx [T, top + nshared] int32, weights fp32)
std::vector<Tensor> moe_route(const Tensor& logits, const Tensor& correction, int64_t top, int64_t nshared, int64_t gate_col,
                              int64_t nslab) {
  TORCH_CHECK(logits.is_cuda() && is_f32(logits), "moe_route: fp32 logits");
  rows(logits, "moe_route");
  f32c(correction, "moe_route correction");
  TORCH_CHECK(nslab >= 1 && logits.size(0) % nslab == 0, "moe_route: slabs");
  const int64_t T = logits.size(0) / nslab, E = correction.numel();
  TORCH_CHECK(logits.size(1) >= E && gate_col < logits.size(1), "moe_route: columns");
  Tensor idx = at::empty({T, top + nshared}, logits.options().dtype(at::kInt));
  Tensor wt = at::empty({T, top + nshared}, logits.options());
  rc_ok(rt_moe_route(logits.data_ptr<float>(), logits.stride(0), (int)nslab, T * logits.stride(0), correction.data_ptr<float>(),
                     (int)T, (int)E, (int)top, (int)nshared, (int)gate_col, idx.data_ptr<int>(), wt.data_ptr<float>(), stream()),
        "moe_route");
  return {idx, wt};
}

// idx [T, slots] with groups in [0, G) -> (offs [G + 1], row_tok [T * slots], pair_pos [T * slots][,
// tiles int32 [max_tiles, 4], n_tiles]) (tile_rows > 0)
std::vector<Tensor> moe_sort(const Tensor& idx, int64_t G, int64_t tile_rows) {
  ints(idx, "moe_sort idx");
  TORCH_CHECK(idx.dim() == 2 && G >= 1 && G <= 1024, "moe_sort: idx [T, slots]");
  const int64_t P = idx.numel();
  Tensor offs = at::empty({G + 1}, idx.options()), tok = at::empty({P}, idx.options()), pos = at::empty({P}, idx.options());
  std::vector<Tensor> r{offs, tok, pos};
  int64_t mt = 0;
  if (tile_rows > 0) {
    mt = P / tile_rows + std::min(G, P);
    r.push_back(at::empty({mt, 4}, idx.options()));
    r.push_back(at::empty({1}, idx.options()));
  }
  rc_ok(rt_moe_sort(idx.data_ptr<int>(), (int)P, (int)idx.size(1), (int)G, offs.data_ptr<int>(), tok.data_ptr<int>(),
                    pos.data_ptr<int>(), (int)tile_rows, (int)mt, tile_rows > 0 ? r[3].data_ptr() : nullptr,
                    tile_rows > 0 ? r[4].data_ptr<int>() : nullptr, stream()),
        "moe_sort");
  return r;
}

// rows of a sorted by group times w [G, N or 2N, K] (glu given: [gate; up] with the gated unit)
Tensor moe_rows(const Tensor& a, const optional<Tensor>& row_map, const Tensor& w, const Tensor& offs, int64_t n_rows,
                bool out_f32, int64_t mean_rows, bool ring, const std::vector<double>& glu) {
  TORCH_CHECK(a.is_cuda() && a.scalar_type() == at::kBFloat16 && w.scalar_type() == at::kBFloat16 && w.is_cuda(), "moe_rows: bf16");
  rows(a, "moe_rows");
  ints(offs, "moe_rows offs");
  const bool pair = !glu.empty();
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous() && w.size(2) == a.size(1) && offs.numel() == w.size(0) + 1 && al16(a) && al16(w),
              "moe_rows: shapes");
  if (has(row_map)) {
    ints(*row_map, "moe_rows row_map");
    TORCH_CHECK(row_map->numel() == n_rows, "moe_rows: row_map");
  } else {
    TORCH_CHECK(a.size(0) == n_rows, "moe_rows: rows");
  }
  const int64_t G = w.size(0), K = w.size(2), N = pair ? w.size(1) / 2 : w.size(1);
  Tensor c = at::empty({n_rows, N}, a.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  float g[3];
  if (pair) for (int i = 0; i < 3; ++i) g[i] = Glu(glu).v[i];
  rc_ok(rt_moe_rows(a.data_ptr(), a.stride(0), (const int*)ptr(row_map), w.data_ptr(), w.stride(0), w.stride(1), c.data_ptr(),
                    N, offs.data_ptr<int>(), (int)G, (int)N, (int)K, pair, out_f32, (int)mean_rows, ring, pair ? g : nullptr, stream()),
        "moe_rows");
  return c;
}

// the same product over 256-row tiles (token-parallel MFMA GEMM)
Tensor gemm_grouped(const Tensor& a, const optional<Tensor>& row_map, const Tensor& w, const Tensor& tiles,
                    const Tensor& n_tiles, int64_t n_rows, const std::vector<double>& glu, int64_t bn) {
  TORCH_CHECK(a.is_cuda() && a.scalar_type() == at::kBFloat16 && w.scalar_type() == at::kBFloat16 && w.is_cuda(), "gemm_grouped: bf16");
  rows(a, "gemm_grouped");
  ints(tiles, "gemm_grouped tiles");
  ints(n_tiles, "gemm_grouped n_tiles");
  const bool pair = !glu.empty();
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous() && w.size(2) == a.size(1) && a.stride(0) % 8 == 0 && al16(a) && al16(w) &&
                  tiles.dim() == 2 && tiles.size(1) == 4, "gemm_grouped: shapes");
  if (has(row_map)) {
    ints(*row_map, "gemm_grouped row_map");
    TORCH_CHECK(row_map->numel() == n_rows, "gemm_grouped: row_map");
  } else {
    TORCH_CHECK(a.size(0) == n_rows, "gemm_grouped: rows");
  }
  const int64_t K = w.size(2), N = w.size(1), Nout = pair ? N / 2 : N;
  TORCH_CHECK(Nout % 8 == 0, "gemm_grouped: output width % 8");
  Tensor c = at::empty({n_rows, Nout}, a.options());
  float g[3];
  if (pair) for (int i = 0; i < 3; ++i) g[i] = Glu(glu).v[i];
  rc_ok(rt_gemm_grouped(a.data_ptr(), a.stride(0), (const int*)ptr(row_map), w.data_ptr(), w.stride(0), w.stride(1), c.data_ptr(),
                        Nout, tiles.data_ptr(), n_tiles.data_ptr<int>(), (int)tiles.size(0), (int)N, (int)K, pair ? 5 : 0,
                        pair ? g : nullptr, zero_page(a).data_ptr(), (int)bn, stream()),
        "gemm_grouped");
  return c;
}

struct Pool {  // pool [pages, 64, KD], table [rows, max_pages]
  const Tensor& pool; const Tensor& tab;
  Pool(const Tensor& p, const Tensor& t) : pool(p), tab(t) {
    act_type(p, "latent pool");
    ints(t, "latent page table");
    TORCH_CHECK(p.dim() == 3 && p.size(1) == 64 && p.is_contiguous() && t.dim() == 2 && al16(p), "latent pool [pages, 64, KD]");
  }
  int pages() const { return (int)pool.size(0); }
  int rows() const { return (int)tab.size(0); }
  int max_pages() const { return (int)tab.size(1); }
  int kd() const { return (int)pool.size(2); }
};

void tok_index(const Tensor& row, const Tensor& pos, int64_t T) {
  ints(row, "latent rows");
  ints(pos, "latent positions");
  TORCH_CHECK(row.numel() >= T && pos.numel() >= T, "latent: one row / position per token");
}

void latent_prep(Tensor proj, int64_t kv_col, const optional<Tensor>& norm_w, double eps, const Tensor& cosT,
                 const Tensor& sinT, const Tensor& row, const Tensor& pos, Tensor pool, const Tensor& tab,
                 const optional<Tensor>& qabs, int64_t n_abs, int64_t H, int64_t dim, int64_t rot, int64_t rank) {
  Pool pl(pool, tab);
  rows(proj, "latent_prep proj");
  same(pool, proj, "latent_prep");
  const int64_t T = proj.size(0);
  tok_index(row, pos, T);
  f32c(cosT, "cos");
  f32c(sinT, "sin");
  TORCH_CHECK(cosT.dim() == 2 && cosT.sizes() == sinT.sizes() && pl.kd() == rank + rot && H * (dim + rot) <= proj.size(1) &&
                  cosT.size(0) >= 1, "latent_prep: shapes");
  TORCH_CHECK(n_abs >= 0 && n_abs <= T, "latent_prep: n_abs");
  if (kv_col >= 0) {
    TORCH_CHECK(kv_col + rank + rot <= proj.size(1) && has(norm_w) && norm_w->numel() == rank && norm_w->is_contiguous(),
                "latent_prep: latent columns");
    same(pool, *norm_w, "latent_prep norm");
  }
  if (n_abs > 0) {
    TORCH_CHECK(has(qabs) && qabs->is_contiguous() && qabs->numel() >= n_abs * H * (rank + rot), "latent_prep: qabs");
    same(pool, *qabs, "latent_prep qabs");
  }
  rc_ok(rt_latent_prep(is_f32(pool), proj.data_ptr(), proj.stride(0), (int)kv_col, ptr(norm_w), (float)eps,
                       cosT.data_ptr<float>(), sinT.data_ptr<float>(), (int)cosT.size(0), (int)cosT.size(1) * 2,
                       row.data_ptr<int>(), pos.data_ptr<int>(), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(),
                       pl.pages(), pl.rows(), ptr(qabs), (int)n_abs, (int)T, (int)H, (int)dim, (int)rot, (int)rank, stream()),
        "latent_prep");
}

// q [T, H, KD] -> (partial latent sums [T, H, NP, rank], (max, sum) [T, H, NP, 2])
std::vector<Tensor> latent_decode(const Tensor& q, const Tensor& pool, const Tensor& tab, const Tensor& row,
                                  const Tensor& pos, int64_t rank, int64_t NP, double scale) {
  Pool pl(pool, tab);
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.scalar_type() == at::kBFloat16 && pool.scalar_type() == at::kBFloat16 &&
                  q.is_cuda() && q.size(2) == pl.kd() && rank <= pl.kd() && NP >= 1 && al16(q), "latent_decode: shapes");
  const int64_t T = q.size(0), H = q.size(1);
  tok_index(row, pos, T);
  Tensor part = at::empty({T, H, NP, rank}, q.options().dtype(at::kFloat));
  Tensor ml = at::empty({T, H, NP, 2}, q.options().dtype(at::kFloat));
  rc_ok(rt_latent_decode(q.data_ptr(), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(), pl.pages(), pl.rows(),
                         row.data_ptr<int>(), pos.data_ptr<int>(), part.data_ptr<float>(), ml.data_ptr<float>(), (int)T,
                         (int)H, (int)rank, pl.kd(), (int)NP, (float)scale, stream()),
        "latent_decode");
  return {part, ml};
}

// partitions -> latent outputs [T, H, rank] (softmax with the sink)
Tensor latent_merge(const Tensor& part, const Tensor& ml, const Tensor& sink) {
  f32c(part, "latent_merge part");
  f32c(ml, "latent_merge ml");
  f32c(sink, "latent_merge sink");
  TORCH_CHECK(part.dim() == 4, "latent_merge: part [T, H, NP, rank]");
  const int64_t T = part.size(0), H = part.size(1), NP = part.size(2), rank = part.size(3);
  TORCH_CHECK(sink.numel() == H && ml.numel() == T * H * NP * 2, "latent_merge: shapes");
  Tensor o = at::empty({T, H, rank}, part.options().dtype(at::kBFloat16));
  rc_ok(rt_partition_merge(part.data_ptr<float>(), ml.data_ptr<float>(), sink.data_ptr<float>(), o.data_ptr(), H * rank, (int)T,
                           (int)H, (int)rank, (int)NP, 1.f, stream()),
        "latent_merge");
  return o;
}

Tensor latent_gather(const Tensor& pool, const Tensor& tab, const Tensor& segs, int64_t total, int64_t max_kv) {
  Pool pl(pool, tab);
  ints(segs, "latent_gather segs");
  TORCH_CHECK(segs.dim() == 2 && segs.size(1) == 8, "latent_gather: segs [S, 8]");
  Tensor out = at::empty({total, pl.kd()}, pool.options());
  rc_ok(rt_latent_gather(is_f32(pool), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(), pl.pages(), segs.data_ptr(),
                         (int)segs.size(0), (int)max_kv, out.data_ptr(), pl.kd(), stream()),
        "latent_gather");
  return out;
}

// q / gate / out rows are the batch's tokens (segments index them); kv [rows, H (dim + vdim) + rot]: unrotated
// keys, values, shared rotated key part
void latent_prefill(const Tensor& q, const Tensor& kv, const Tensor& sink, const Tensor& gate, Tensor out,
                    const Tensor& segs, const Tensor& tiles, int64_t H, int64_t dim, int64_t rot, int64_t vdim, double scale) {
  for (const Tensor* t : {&q, &kv, &gate}) {
    rows(*t, "latent_prefill");
    TORCH_CHECK(t->is_cuda() && t->scalar_type() == at::kBFloat16 && al16(*t), "latent_prefill: bf16 rows, 16-B aligned");
  }
  rows(out, "latent_prefill out");
  TORCH_CHECK(out.scalar_type() == at::kBFloat16 && al16(out), "latent_prefill: out");
  ints(segs, "segs");
  ints(tiles, "tiles");
  f32c(sink, "sink");
  TORCH_CHECK(segs.dim() == 2 && segs.size(1) == 8 && tiles.dim() == 2 && tiles.size(1) == 2, "latent_prefill: tables");
  TORCH_CHECK(q.size(1) >= H * (dim + rot) && kv.size(1) == H * (dim + vdim) + rot && gate.size(1) == H * vdim &&
                  out.size(1) == H * vdim && sink.numel() == H, "latent_prefill: shapes");
  rc_ok(rt_latent_prefill(q.data_ptr(), q.stride(0), kv.data_ptr(), kv.stride(0), (int)(H * dim), (int)(H * (dim + vdim)),
                          sink.data_ptr<float>(), gate.data_ptr(), gate.stride(0), out.data_ptr(), out.stride(0),
                          segs.data_ptr(), tiles.data_ptr(), (int)tiles.size(0), (int)H, (int)dim, (int)rot, (int)vdim,
                          (float)scale, stream()),
        "latent_prefill");
}

// q [T, H, KD] -> latent outputs [T, H, rank] (softmax with the sink), any size, bf16 / fp32
Tensor latent_any(const Tensor& q, const Tensor& pool, const Tensor& tab, const Tensor& row, const Tensor& pos,
                  const Tensor& sink, int64_t rank, double scale) {
  Pool pl(pool, tab);
  same(pool, q, "latent_any");
  f32c(sink, "sink");
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.size(2) == pl.kd() && rank <= pl.kd() && sink.numel() == q.size(1),
              "latent_any: shapes");
  tok_index(row, pos, q.size(0));
  Tensor o = at::empty({q.size(0), q.size(1), rank}, q.options());
  rc_ok(rt_latent_any(is_f32(pool), q.data_ptr(), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(), pl.pages(), pl.rows(),
                      row.data_ptr<int>(), pos.data_ptr<int>(), sink.data_ptr<float>(), o.data_ptr(), (int)q.size(0),
                      (int)q.size(1), (int)rank, pl.kd(), (float)scale, stream()),
        "latent_any");
  return o;
}

// ---- grouped-query attention over a paged window ----
// pool [pages, 64, G (D + V)] (inside a page: [G][64][D + V])
struct Win {
  int H, G, D, V, size, keep;
  float scale, cap;
  // {heads, key heads, key width, value width, window (0: none), kept first tokens}, {scale, softcap (0: none)}
  Win(const std::vector<int64_t>& d, const std::vector<double>& f, const Pool& pl) {
    TORCH_CHECK(d.size() == 6 && f.size() == 2, "window attention: dims {6}, {2}");
    H = (int)d[0]; G = (int)d[1]; D = (int)d[2]; V = (int)d[3]; size = (int)d[4]; keep = (int)d[5];
    scale = (float)f[0]; cap = (float)f[1];
    TORCH_CHECK(H > 0 && G > 0 && H % G == 0 && D > 0 && V > 0 && size >= 0 && keep >= 0 && pl.kd() == G * (D + V) &&
                    pl.rows() > 0 && pl.max_pages() > 0, "window attention: sizes");
  }
};

// proj [N, ..] = q | k | v from column col: q normed and rotated in place, k and v to the cache
void window_prep(Tensor proj, int64_t col, const optional<Tensor>& q_norm, const optional<Tensor>& k_norm, double eps,
                 const Tensor& cosT, const Tensor& sinT, const Tensor& row, const Tensor& pos, Tensor pool, const Tensor& tab,
                 const std::vector<int64_t>& dims, const std::vector<double>& fs) {
  Pool pl(pool, tab);
  const Win w(dims, fs, pl);
  rows(proj, "window_prep proj");
  same(pool, proj, "window_prep");
  const int64_t T = proj.size(0), nq = (int64_t)w.H * w.D, nk = (int64_t)w.G * w.D;
  tok_index(row, pos, T);
  f32c(cosT, "cos");
  f32c(sinT, "sin");
  TORCH_CHECK(cosT.dim() == 2 && cosT.sizes() == sinT.sizes() && cosT.size(0) >= 1 && 2 * cosT.size(1) <= w.D && col >= 0 &&
                  col + nq + nk + (int64_t)w.G * w.V <= proj.size(1), "window_prep: shapes");
  if (has(q_norm)) {
    same(pool, *q_norm, "window_prep q norm");
    TORCH_CHECK(q_norm->is_contiguous() && q_norm->numel() == nq, "window_prep: q norm");
  }
  if (has(k_norm)) {
    same(pool, *k_norm, "window_prep k norm");
    TORCH_CHECK(k_norm->is_contiguous() && k_norm->numel() == nk, "window_prep: k norm");
  }
  rc_ok(rt_window_prep(is_f32(pool), proj.data_ptr(), proj.stride(0), (int)col, (int)(col + nq), (int)(col + nq + nk), ptr(q_norm),
                       ptr(k_norm), (float)eps, cosT.data_ptr<float>(), sinT.data_ptr<float>(), (int)cosT.size(0),
                       (int)cosT.size(1), row.data_ptr<int>(), pos.data_ptr<int>(), pool.data_ptr(), tab.data_ptr<int>(),
                       pl.max_pages(), pl.pages(), pl.rows(), (int)T, w.H, w.G, w.D, w.V, stream()),
        "window_prep");
}

// tokens [0, T) of q [.., H D] and out [.., H V] (strided rows), keys and values from the cache
void window_decode(const Tensor& q, const Tensor& pool, const Tensor& tab, const Tensor& row, const Tensor& pos, Tensor out,
                   int64_t NP, double out_scale, const std::vector<int64_t>& dims, const std::vector<double>& fs) {
  Pool pl(pool, tab);
  const Win w(dims, fs, pl);
  rows(q, "window_decode q");
  rows(out, "window_decode out");
  const int64_t T = q.size(0);
  tok_index(row, pos, T);
  TORCH_CHECK(pool.scalar_type() == at::kBFloat16 && q.scalar_type() == at::kBFloat16 && out.scalar_type() == at::kBFloat16 &&
                  q.is_cuda() && out.is_cuda() && q.size(1) == (int64_t)w.H * w.D && out.size(0) == T &&
                  out.size(1) == (int64_t)w.H * w.V && NP >= 1 && NP <= 1024 && al16(q), "window_decode: shapes");
  Tensor part = at::empty({T, w.H, NP, w.V}, q.options().dtype(at::kFloat));
  Tensor ml = at::empty({T, w.H, NP, 2}, q.options().dtype(at::kFloat));
  rc_ok(rt_window_decode(q.data_ptr(), q.stride(0), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(), pl.pages(), pl.rows(),
                         row.data_ptr<int>(), pos.data_ptr<int>(), part.data_ptr<float>(), ml.data_ptr<float>(), (int)T, w.H, w.G,
                         w.D, w.V, (int)NP, w.size, w.keep, w.scale, w.cap, stream()),
        "window_decode");
  rc_ok(rt_partition_merge(part.data_ptr<float>(), ml.data_ptr<float>(), nullptr, out.data_ptr(), out.stride(0), (int)T, w.H, w.V,
                           (int)NP, (float)out_scale, stream()),
        "partition_merge");
}

void window_prefill(const Tensor& q, const Tensor& pool, const Tensor& tab, Tensor out, const Tensor& segs, const Tensor& tiles,
                    double out_scale, const std::vector<int64_t>& dims, const std::vector<double>& fs) {
  Pool pl(pool, tab);
  const Win w(dims, fs, pl);
  rows(q, "window_prefill q");
  rows(out, "window_prefill out");
  ints(segs, "segs");
  ints(tiles, "tiles");
  TORCH_CHECK(pool.scalar_type() == at::kBFloat16 && q.scalar_type() == at::kBFloat16 && out.scalar_type() == at::kBFloat16 &&
                  q.is_cuda() && out.is_cuda() && q.size(1) == (int64_t)w.H * w.D && out.size(0) == q.size(0) &&
                  out.size(1) == (int64_t)w.H * w.V && al16(q) && segs.dim() == 2 && segs.size(1) == 8 && tiles.dim() == 2 &&
                  tiles.size(1) == 2, "window_prefill: shapes");
  rc_ok(rt_window_prefill(q.data_ptr(), q.stride(0), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(), pl.pages(), pl.rows(),
                          out.data_ptr(), out.stride(0), segs.data_ptr(), tiles.data_ptr(), (int)tiles.size(0), w.H, w.G, w.D,
                          w.V, w.size, w.keep, w.scale, w.cap, (float)out_scale, stream()),
        "window_prefill");
}

void window_any(const Tensor& q, const Tensor& pool, const Tensor& tab, const Tensor& row, const Tensor& pos, Tensor out,
                double out_scale, const std::vector<int64_t>& dims, const std::vector<double>& fs) {
  Pool pl(pool, tab);
  const Win w(dims, fs, pl);
  rows(q, "window_any q");
  rows(out, "window_any out");
  same(pool, q, "window_any");
  same(pool, out, "window_any");
  tok_index(row, pos, q.size(0));
  TORCH_CHECK(q.size(1) == (int64_t)w.H * w.D && out.size(0) == q.size(0) && out.size(1) == (int64_t)w.H * w.V, "window_any: shapes");
  rc_ok(rt_window_any(is_f32(pool), q.data_ptr(), q.stride(0), pool.data_ptr(), tab.data_ptr<int>(), pl.max_pages(), pl.pages(),
                      pl.rows(), row.data_ptr<int>(), pos.data_ptr<int>(), out.data_ptr(), out.stride(0), (int)q.size(0), w.H,
                      w.G, w.D, w.V, w.size, w.keep, w.scale, w.cap, (float)out_scale, stream()),
        "window_any");
}

// ---- gated delta rule ----
// x [N, C] (q | k | v projections), b [N, H], a [N, H or H D], z [N, H V], out [N, H V]: strided rows of one
// type; S [rows, H, D, V] fp32, ring [rows, taps, C]. Tokens [0, n_single): one per request; the rest by runs
// [R, 4] {row, first token, tokens, position}, chunks [.., 2] {run, chunk}, first_chunk [R].
void delta_rule(const Tensor& x, const Tensor& b, const Tensor& a, const Tensor& z, const Tensor& conv, const Tensor& A_log,
                const Tensor& dt, const Tensor& norm_w, double eps, const Tensor& row, const Tensor& pos, Tensor S, Tensor ring,
                Tensor out, double out_scale, int64_t K, bool silu, int64_t n_single, const optional<Tensor>& runs,
                const optional<Tensor>& chunks, const optional<Tensor>& first_chunk) {
  act_type(x, "delta_rule x");
  for (const Tensor* t : {&x, &b, &a, &z, (const Tensor*)&out}) {
    rows(*t, "delta_rule rows");
    same(x, *t, "delta_rule");
    TORCH_CHECK(t->size(0) == x.size(0), "delta_rule: one row per token");
  }
  f32c(S, "delta_rule state");
  f32c(A_log, "delta_rule A_log");
  f32c(dt, "delta_rule dt");
  same(x, ring, "delta_rule ring");
  same(x, conv, "delta_rule conv");
  same(x, norm_w, "delta_rule norm");
  const int64_t N = x.size(0);
  TORCH_CHECK(S.dim() == 4 && S.size(0) >= 1, "delta_rule: S [rows, H, D, V]");
  const int64_t H = S.size(1), D = S.size(2), V = S.size(3), C = x.size(1);
  TORCH_CHECK(K >= 1 && H % K == 0 && C == 2 * K * D + H * V && conv.dim() == 2 && conv.size(0) == C && conv.is_contiguous() &&
                  conv.size(1) >= 1, "delta_rule: channels");
  const int64_t taps = conv.size(1);
  const bool channel = dt.numel() == H * D && a.size(1) == H * D && !(D == 1);
  TORCH_CHECK(A_log.numel() == H && (channel || (dt.numel() == H && a.size(1) == H)) && b.size(1) == H && z.size(1) == H * V &&
                  out.size(1) == H * V && norm_w.numel() == V && norm_w.is_contiguous(), "delta_rule: shapes");
  TORCH_CHECK(ring.dim() == 3 && ring.size(0) == S.size(0) && ring.size(1) == taps && ring.size(2) == C && ring.is_contiguous(),
              "delta_rule: ring [rows, taps, C]");
  tok_index(row, pos, N);
  TORCH_CHECK(n_single >= 0 && n_single <= N && (n_single == N || has(runs)), "delta_rule: runs");
  RtDelta d{x.data_ptr(), x.stride(0), b.data_ptr(), b.stride(0), a.data_ptr(), a.stride(0), z.data_ptr(), z.stride(0),
            conv.data_ptr(), A_log.data_ptr<float>(), dt.data_ptr<float>(), norm_w.data_ptr(), (float)eps, row.data_ptr<int>(),
            pos.data_ptr<int>(), S.data_ptr<float>(), ring.data_ptr(), (int)S.size(0), out.data_ptr(), out.stride(0),
            (float)out_scale, (int)H, (int)K, (int)D, (int)V, (int)taps, channel, silu};
  rc_ok(rt_delta_step(is_f32(x), &d, (int)n_single, stream()), "delta_step");
  if (n_single == N) return;
  ints(*runs, "delta_rule runs");
  TORCH_CHECK(has(chunks) && has(first_chunk), "delta_rule: chunks");
  ints(*chunks, "delta_rule chunks");
  ints(*first_chunk, "delta_rule first_chunk");
  TORCH_CHECK(runs->dim() == 2 && runs->size(1) == 4 && chunks->dim() == 2 && chunks->size(1) == 2 && first_chunk->numel() == runs->size(0) &&
                  al16(*runs) && reinterpret_cast<uintptr_t>(chunks->data_ptr()) % 8 == 0, "delta_rule: tables");
  const long per = rt_delta_ws((int)D);
  TORCH_CHECK(per > 0, "delta_rule: key width ", D, " above 256");
  Tensor ws = at::empty({chunks->size(0) * H * per}, x.options().dtype(at::kFloat));
  Tensor v = at::empty({N, (H * V + 1) / 2 * 2}, x.options()), o = at::empty({N, H * V}, x.options().dtype(at::kFloat));
  rc_ok(rt_delta_runs(is_f32(x), &d, runs->data_ptr(), chunks->data_ptr(), first_chunk->data_ptr<int>(), (int)runs->size(0),
                      (int)chunks->size(0), (int)n_single, (int)(N - n_single), ws.data_ptr<float>(), v.data_ptr(),
                      o.data_ptr<float>(), stream()),
        "delta_runs");
}

}  // namespace

void bind_layered(py::module_& m) {
  m.def("branch_norm", &branch_norm, "x += rms(y) w_branch; h = rms(x) w_next (fp32 residual)", py::arg("x"), py::arg("kind"),
        py::arg("y") = py::none(), py::arg("nsplit") = 1, py::arg("w_branch") = py::none(), py::arg("w_next") = py::none(),
        py::arg("table") = py::none(), py::arg("ids") = py::none(), py::arg("pair_w") = py::none(),
        py::arg("pair_pos") = py::none(), py::arg("eps"), py::arg("scale") = py::none(), py::arg("next_mul") = 1.0,
        py::arg("plain") = false);
  m.def("gemm_any", &gemm_any, "a w^T, any shape, bf16 / fp32, batched or grouped", py::arg("a"), py::arg("w"),
        py::arg("out_f32") = false, py::arg("out") = py::none(), py::arg("offs") = py::none(), py::arg("row_map") = py::none());
  m.def("head_gemm", &head_gemm, "per-head a w^T at few rows (gated)", py::arg("a"), py::arg("w"), py::arg("out"),
        py::arg("gate") = py::none());
  m.def("glu_any", &glu_any, "gated linear unit of [gate | up] rows");
  m.def("act_any", &act_any, "activation of an fp32 product");
  m.def("gate_mul", &gate_mul, "a *= sigmoid(g)");
  m.def("moe_route", &moe_route, "softmax router with choice correction -> experts, weights", py::arg("logits"),
        py::arg("correction"), py::arg("top"), py::arg("nshared"), py::arg("gate_col"), py::arg("nslab") = 1);
  m.def("moe_sort", &moe_sort, "stable sort of (token, slot) pairs by expert");
  m.def("moe_rows", &moe_rows, "grouped product at few rows per group");
  m.def("gemm_grouped", &gemm_grouped, "grouped product over 256-row tiles");
  m.def("latent_prep", &latent_prep, "latent norm, rotation, cache append");
  m.def("latent_decode_ok", [](int rank, int kd) { return rt_latent_decode_ok(rank, kd) != 0; });
  m.def("latent_prefill_ok", [](int dim, int rot, int vdim) { return rt_latent_prefill_ok(dim, rot, vdim) != 0; });
  m.def("latent_decode", &latent_decode, "absorbed attention partials over the paged latent cache");
  m.def("latent_merge", &latent_merge, "partition merge with the sink");
  m.def("latent_gather", &latent_gather, "cached rows of each segment, dense");
  m.def("latent_prefill", &latent_prefill, "flash attention of prompt portions over expanded keys / values");
  m.def("window_prep", &window_prep, "q / k norm, rotation in halves, cache append");
  m.def("window_decode_ok", [](int H, int G, int D, int V) { return rt_window_decode_ok(H, G, D, V) != 0; });
  m.def("window_prefill_ok", [](int D, int V) { return rt_window_prefill_ok(D, V) != 0; });
  m.def("window_decode", &window_decode, "windowed attention, few tokens per request");
  m.def("window_prefill", &window_prefill, "windowed flash attention of prompt portions from the pages");
  m.def("window_any", &window_any, "windowed attention, any size / type");
  m.def("delta_rule", &delta_rule, "gated delta rule over a ragged batch");
  m.def("latent_any", &latent_any, "absorbed attention, any size / type");
}
