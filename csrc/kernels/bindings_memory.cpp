// torch operator registrations (namespace torch.ops.dsse) of the kernels in api_memory.h: the convolved / rotated q | k | v
// rows, the matrix memory and the work lists of table-routed experts.
//
// As in the other binding files, every op validates device, dtype and the shapes and strides its kernel's indexing
// assumes before launching, and launches on torch's current HIP stream (graph-capturable).
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <torch/library.h>

#include <algorithm>
#include <climits>
#include <cstdint>

#include "api_memory.h"

namespace {

using at::Tensor;
using OptTensor = c10::optional<Tensor>;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define DSSE_CHECK_HIP(expr)                                                             \
  do {                                                                                   \
    hipError_t _e = (expr);                                                              \
    TORCH_CHECK(_e == hipSuccess, "dsse kernel launch failed: ", hipGetErrorString(_e)); \
  } while (0)

void gpu(const Tensor& t, const char* name, bool contiguous = true) {
  TORCH_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  if (contiguous) TORCH_CHECK(t.is_contiguous(), name, " must be contiguous");
}
void i32(const Tensor& t, const char* name) {
  gpu(t, name);
  TORCH_CHECK(t.scalar_type() == at::kInt, name, " must be int32");
}
void f32t(const Tensor& t, const char* name, bool contiguous = true) {
  gpu(t, name, contiguous);
  TORCH_CHECK(t.scalar_type() == at::kFloat, name, " must be fp32");
}
int elem(const Tensor& a, const char* name) {
  TORCH_CHECK(a.scalar_type() == at::kFloat || a.scalar_type() == at::kBFloat16, name, " must be bf16 or fp32");
  return a.scalar_type() == at::kFloat ? 1 : 0;
}
// a [rows, heads, width] fp32 view whose heads are adjacent columns of a row-major buffer
void head_view(const Tensor& t, const char* name) {
  f32t(t, name, false);
  TORCH_CHECK(t.dim() == 3 && (t.size(2) == 1 || t.stride(2) == 1) && (t.size(1) == 1 || t.stride(1) == t.size(2)) &&
                  t.stride(0) >= t.size(1) * t.size(2) && t.stride(0) < INT_MAX,
              name, " must be [rows, heads, width] with adjacent heads");
}
// a [rows, cols] view with a unit innermost stride
void col_view(const Tensor& t, const char* name) {
  gpu(t, name, false);
  TORCH_CHECK(t.dim() == 2 && (t.size(1) == 1 || t.stride(1) == 1) && t.stride(0) >= t.size(1) && t.stride(0) < INT_MAX, name,
              " must be [rows, cols] with a unit innermost stride");
}
int seq_meta(const Tensor& q_start, const Tensor& q_len, const Tensor& ctx_len, const Tensor& state_slot) {
  i32(q_start, "q_start");
  i32(q_len, "q_len");
  i32(ctx_len, "ctx_len");
  i32(state_slot, "state_slot");
  const int64_t n = q_len.numel();
  TORCH_CHECK(q_start.numel() >= n && ctx_len.numel() >= n && state_slot.numel() >= n && n <= 65535,
              "sequence metadata lengths");
  return (int)n;
}
bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

void conv_qkv_rows(const Tensor& x, const OptTensor& taps, const OptTensor& tail, const Tensor& q_start, const Tensor& q_len,
                   const Tensor& ctx_len, const Tensor& state_slot, const Tensor& work_seq, const Tensor& work_tile,
                   int64_t qt, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, const OptTensor& rope,
                   const OptTensor& q_factor, const Tensor& slots, Tensor& q, Tensor& kcache, Tensor& vcache,
                   const OptTensor& vt) {
  col_view(x, "x");
  f32t(x, "x", false);
  f32t(q, "q");
  dsse::ConvQkvParams p{};
  const int64_t T = x.size(0);
  TORCH_CHECK(heads >= 1 && kv_heads >= 1 && dim >= 1 && vdim >= 0 && dim <= 512 && vdim <= 512 && qt >= 1 &&
                  heads <= 65535 && kv_heads <= 65535,
              "head counts and widths");
  p.H = (int)heads, p.G = (int)kv_heads, p.D = (int)dim, p.V = (int)vdim, p.qt = (int)qt;
  const int64_t C = (heads + kv_heads) * dim, VW = vdim == 0 ? dim : vdim;
  TORCH_CHECK(x.size(1) >= C + kv_heads * vdim, "x must hold the q | k | v columns");
  TORCH_CHECK(q.dim() == 3 && q.size(0) == T && q.size(1) == heads && q.size(2) == dim, "q must be [T, H, D]");
  p.nseq = seq_meta(q_start, q_len, ctx_len, state_slot);
  i32(work_seq, "work_seq");
  i32(work_tile, "work_tile");
  TORCH_CHECK(work_seq.numel() == work_tile.numel() && work_seq.numel() <= 65535, "work lists");
  p.nwork = (int)work_seq.numel();
  if (taps.has_value()) {
    f32t(*taps, "taps");
    TORCH_CHECK(taps->dim() == 2 && taps->size(0) == C && taps->size(1) >= 1 && taps->size(1) <= 64,
                "taps must be [(H + G) D, K]");
    p.K = (int)taps->size(1);
    p.taps = taps->data_ptr<float>();
    if (p.K > 1) {
      TORCH_CHECK(tail.has_value(), "a convolution with more than one tap needs its tail");
      f32t(*tail, "tail");
      TORCH_CHECK(tail->dim() == 3 && tail->size(1) == p.K - 1 && tail->size(2) == C, "tail must be [slots, K - 1, (H + G) D]");
      p.tail = tail->data_ptr<float>();
    }
  }
  if (rope.has_value() && rope->numel() > 0) {
    f32t(*rope, "rope");
    TORCH_CHECK(rope->dim() == 3 && rope->size(2) == 2 && 2 * rope->size(1) <= dim && rope->size(0) < INT_MAX,
                "rope must be [P, dims / 2, 2]");
    p.rope = reinterpret_cast<const float2*>(rope->data_ptr<float>());
    p.half = (int)rope->size(1), p.rope_len = (int)rope->size(0);
  }
  if (q_factor.has_value()) {
    f32t(*q_factor, "q_factor");
    TORCH_CHECK(q_factor->dim() == 1 && q_factor->numel() >= 1 && q_factor->numel() < INT_MAX, "q_factor must be [P]");
    p.q_factor = q_factor->data_ptr<float>();
    p.q_factor_len = (int)q_factor->numel();
  }
  i32(slots, "slots");
  TORCH_CHECK(slots.numel() >= T, "slots too short");
  gpu(kcache, "kcache");
  gpu(vcache, "vcache");
  TORCH_CHECK(kcache.dim() == 4 && vcache.dim() == 4 && kcache.scalar_type() == vcache.scalar_type() &&
                  kcache.size(1) == dsse::kBS && vcache.size(1) == dsse::kBS && kcache.size(2) == kv_heads &&
                  vcache.size(2) == kv_heads && kcache.size(3) == dim && vcache.size(3) == VW &&
                  kcache.size(0) == vcache.size(0) && kcache.size(0) * dsse::kBS < INT_MAX,
              "caches must be [pages, 32, G, D] and [pages, 32, G, V]");
  p.f32 = elem(kcache, "kcache");
  p.num_slots = (int)(kcache.size(0) * dsse::kBS);
  if (vt.has_value()) {
    gpu(*vt, "vt");
    TORCH_CHECK(vt->scalar_type() == vcache.scalar_type() && vt->dim() == 4 && vt->size(0) == vcache.size(0) &&
                    vt->size(1) == kv_heads && vt->size(2) == VW && vt->size(3) == dsse::kBS,
                "vt must be [pages, G, V, 32]");
    p.vt = vt->data_ptr();
  }
  p.x = x.data_ptr<float>();
  p.ldx = (int)x.stride(0);
  p.q_start = q_start.data_ptr<int>();
  p.q_len = q_len.data_ptr<int>();
  p.ctx_len = ctx_len.data_ptr<int>();
  p.state_slot = state_slot.data_ptr<int>();
  p.work_seq = work_seq.data_ptr<int>();
  p.work_tile = work_tile.data_ptr<int>();
  p.slots = slots.data_ptr<int>();
  p.q = q.data_ptr<float>();
  p.k = kcache.data_ptr();
  p.v = vcache.data_ptr();
  DSSE_CHECK_HIP(dsse_conv_qkv_rows(&p, cur_stream()));
}

void matrix_memory(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& gates, const Tensor& gate_b, double cap,
                   Tensor& state, Tensor& norm, const Tensor& q_start, const Tensor& q_len, const Tensor& ctx_len,
                   const Tensor& state_slot, const Tensor& out_gate, const Tensor& norm_w, double eps, double den_eps,
                   double q_scale, double out_scale, Tensor& out, const OptTensor& work, int64_t row0, int64_t rows) {
  head_view(q, "q");
  head_view(k, "k");
  head_view(v, "v");
  col_view(gates, "gates");
  f32t(gates, "gates", false);
  col_view(out_gate, "out_gate");
  f32t(out_gate, "out_gate", false);
  col_view(out, "out");
  f32t(gate_b, "gate_b");
  f32t(norm_w, "norm_w");
  f32t(state, "state");
  f32t(norm, "norm");
  dsse::MatrixMemoryParams p{};
  const int64_t T = v.size(0), H = v.size(1), V = v.size(2), D = k.size(2);
  TORCH_CHECK(q.sizes() == k.sizes() && k.size(0) == T && k.size(1) == H && D >= 1 && D <= 512 && V >= 1 && V <= 512 &&
                  H >= 1 && H <= 65535 && T < INT_MAX,
              "q and k must be [T, H, D], v [T, H, V], widths <= 512");
  TORCH_CHECK(gates.size(0) == T && gates.size(1) == 2 * H && gate_b.numel() == 2 * H, "gates must be [T, 2 H], gate_b [2 H]");
  TORCH_CHECK(out_gate.size(0) == T && out_gate.size(1) == H * V && out.size(0) == T && out.size(1) == H * V &&
                  norm_w.numel() == H * V,
              "out_gate and out must be [T, H V], norm_w [H V]");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == D && state.size(3) == V && norm.dim() == 3 &&
                  norm.size(0) == state.size(0) && norm.size(1) == H && norm.size(2) == D + 1,
              "state must be [slots, H, D, V], norm [slots, H, D + 1]");
  TORCH_CHECK(cap > 0, "cap > 0");
  p.nseq = seq_meta(q_start, q_len, ctx_len, state_slot);
  p.T = (int)T, p.H = (int)H, p.D = (int)D, p.V = (int)V;
  p.q = q.data_ptr<float>(), p.k = k.data_ptr<float>(), p.v = v.data_ptr<float>();
  p.ldq = (int)q.stride(0), p.ldk = (int)k.stride(0), p.ldv = (int)v.stride(0);
  p.gates = gates.data_ptr<float>(), p.ldz = (int)gates.stride(0);
  p.gate_b = gate_b.data_ptr<float>();
  p.state = state.data_ptr<float>(), p.norm = norm.data_ptr<float>();
  p.q_start = q_start.data_ptr<int>(), p.q_len = q_len.data_ptr<int>();
  p.ctx_len = ctx_len.data_ptr<int>(), p.state_slot = state_slot.data_ptr<int>();
  p.out_gate = out_gate.data_ptr<float>(), p.ldg = (int)out_gate.stride(0);
  p.norm_w = norm_w.data_ptr<float>();
  p.out = out.data_ptr(), p.ldo = (int)out.stride(0);
  p.f32 = elem(out, "out");
  p.cap = (float)cap, p.eps = (float)eps, p.den_eps = (float)den_eps, p.q_scale = (float)q_scale;
  p.out_scale = (float)out_scale;
  if (!work.has_value()) {
    DSSE_CHECK_HIP(dsse_matrix_memory_walk(&p, cur_stream()));
    return;
  }
  f32t(*work, "work");
  const int64_t n = T * H;
  TORCH_CHECK(!p.f32 && D <= 256 && D % 4 == 0, "the MFMA form is bf16, D <= 256, D % 4 == 0");
  const int64_t ldsum = ((T + 3) & ~(int64_t)3) + 4 * p.nseq + 4, n4 = (n + 3) & ~(int64_t)3;
  TORCH_CHECK(work->numel() >= 2 * H * ldsum + 2 * n4 + n * V && aligned16(work->data_ptr()), "work area too small");
  TORCH_CHECK(p.ldk < (1 << 24) && p.ldq < (1 << 24) && p.ldv < (1 << 24), "q, k, v rows too far apart");
  TORCH_CHECK(row0 >= 0 && rows >= 0 && row0 + rows <= T && rows * H < INT_MAX, "the rows of the call");
  float* w = work->data_ptr<float>();
  p.acum = w, p.u = w + H * ldsum, p.nq = w + 2 * H * ldsum, p.m = p.nq + n4, p.num = p.m + n4;
  p.ldsum = (int)ldsum;
  p.row0 = (int)row0, p.rows = (int)rows;
  p.vec = aligned16(p.q) && aligned16(p.k) && p.ldq % 4 == 0 && p.ldk % 4 == 0;
  DSSE_CHECK_HIP(dsse_matrix_memory_chunk(&p, cur_stream()));
}

void moe_table_lists(const Tensor& ids, at::TensorList tables, at::IntArrayRef experts, at::IntArrayRef shared,
                     at::TensorList topk_idx, at::TensorList sorted, at::TensorList tile_expert, at::TensorList num_tiles) {
  i32(ids, "ids");
  const size_t L = tables.size();
  TORCH_CHECK(experts.size() == L && shared.size() == L && topk_idx.size() == L && sorted.size() == L &&
                  tile_expert.size() == L && num_tiles.size() == L,
              "one entry per layer");
  for (size_t l0 = 0; l0 < L; l0 += dsse::kTableLayers) {
    dsse::MoeTableListsParams p{};
    p.ids = ids.data_ptr<int>();
    p.layers = (int)std::min<size_t>(L - l0, dsse::kTableLayers);
    p.M = (int)topk_idx[l0].size(0);
    p.vocab = (int)tables[l0].size(0);
    TORCH_CHECK(ids.numel() >= p.M && p.vocab >= 1, "ids too short");
    for (int i = 0; i < p.layers; ++i) {
      const Tensor &t = tables[l0 + i], &k = topk_idx[l0 + i], &s = sorted[l0 + i], &e = tile_expert[l0 + i],
                   &n = num_tiles[l0 + i];
      i32(t, "table");
      i32(k, "topk_idx");
      i32(s, "sorted");
      i32(e, "tile_expert");
      i32(n, "num_tiles");
      TORCH_CHECK(t.dim() == 2 && k.dim() == 2 && t.size(0) == p.vocab && k.size(0) == p.M && k.size(1) == t.size(1) &&
                      t.size(1) >= 1,
                  "tables must be [vocab, top], topk_idx [M, top]");
      auto& y = p.layer[i];
      y.top = (int)t.size(1), y.S = y.top + (shared[l0 + i] ? 1 : 0), y.E = (int)experts[l0 + i];
      y.max_tiles = (int)e.numel();
      TORCH_CHECK(y.E >= 1 && y.E < 4096 && (int64_t)p.M * y.S < INT_MAX &&
                      y.max_tiles >= ((int64_t)p.M * y.S + 63) / 64 + y.E + 1 && s.numel() >= (int64_t)y.max_tiles * 64 &&
                      n.numel() >= 1,
                  "work lists too small");
      y.table = t.data_ptr<int>(), y.topk_idx = k.data_ptr<int>(), y.sorted = s.data_ptr<int>();
      y.tile_expert = e.data_ptr<int>(), y.num_tiles = n.data_ptr<int>();
    }
    DSSE_CHECK_HIP(dsse_moe_table_lists(&p, cur_stream()));
  }
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(dsse, m) {
  m.def("conv_qkv_rows(Tensor x, Tensor? taps, Tensor(a!)? tail, Tensor q_start, Tensor q_len, Tensor ctx_len, "
        "Tensor state_slot, Tensor work_seq, Tensor work_tile, int qt, int heads, int kv_heads, int dim, int vdim, "
        "Tensor? rope, Tensor? q_factor, Tensor slots, Tensor(b!) q, Tensor(c!) kcache, Tensor(d!) vcache, "
        "Tensor(e!)? vt=None) -> ()");
  m.def("matrix_memory(Tensor q, Tensor k, Tensor v, Tensor gates, Tensor gate_b, float cap, Tensor(a!) state, "
        "Tensor(b!) norm, Tensor q_start, Tensor q_len, Tensor ctx_len, Tensor state_slot, Tensor out_gate, Tensor norm_w, "
        "float eps, float den_eps, float q_scale, float out_scale, Tensor(c!) out, Tensor(d!)? work=None, int row0=0, "
        "int rows=0) -> ()");
  m.def("moe_table_lists(Tensor ids, Tensor[] tables, int[] experts, int[] shared, Tensor(a!)[] topk_idx, "
        "Tensor(b!)[] sorted, Tensor(c!)[] tile_expert, Tensor(d!)[] num_tiles) -> ()");
}

TORCH_LIBRARY_IMPL(dsse, CUDA, m) {
  m.impl("conv_qkv_rows", &conv_qkv_rows);
  m.impl("matrix_memory", &matrix_memory);
  m.impl("moe_table_lists", &moe_table_lists);
}
