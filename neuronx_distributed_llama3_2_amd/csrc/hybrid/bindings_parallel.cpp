// Python bindings of the kernels around parallel sublayers: residual sum + grouped norms, the generalised
// delta rule, the router and the routed experts (part of the module of bindings_hybrid.cpp).
#include "bindings_util.h"
#include "channel_delta.h"
#include "experts.h"
#include "group_norm.h"

namespace nxd {
int residual_norms_launch(bool, const GroupNormParams&, bool, hipStream_t);
int channel_delta_chunk(int);
int channel_delta_step_launch(bool, const ChannelDeltaParams&, hipStream_t);
int channel_delta_chunk_launch(bool, const ChannelDeltaParams&, hipStream_t);
int moe_route_chunk();
int moe_route_launch(const RouterParams&, hipStream_t);
int clamped_glu_launch(bool, const GluParams&, bool, hipStream_t);
int gather_rows_launch(const void*, const int*, void*, int64_t, int64_t, int64_t, hipStream_t);
int experts_few_launch(const RouterParams&, const ExpertFewParams&, hipStream_t);
int linear_few_launch(const LinearFewParams&, hipStream_t);
int expert_rows_launch(bool, const ExpertRowsParams&, hipStream_t);
int grouped_gemm_launch(int, const void*, const void*, void*, const int*, int, int, int, int, int, hipStream_t);
int grouped_rowgemm_launch(int, const void*, const void*, void*, const int*, int, int, int, int, hipStream_t);
}  // namespace nxd

namespace {

using namespace nxd::bind;

bool aligned16(const Tensor& t) { return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0; }

void residual_norms(Tensor x, Opt embed, Opt ids, std::vector<Tensor> adds, Opt pairs, Opt inverse, std::vector<Tensor> norms,
                    double eps, int64_t groups, std::vector<Tensor> hs, Opt rows, bool store) {
  TORCH_CHECK(x.dim() == 2 && x.is_cuda() && x.scalar_type() == at::kFloat && x.is_contiguous(), "residual_norms: x fp32 [M, W]");
  nxd::GroupNormParams p{};
  p.M = x.size(0);
  p.W = (int)x.size(1);
  TORCH_CHECK(p.M >= 1 && p.W >= 1 && p.W <= 16384 && groups >= 1 && p.W % groups == 0, "residual_norms: width up to 16384, equal groups");
  TORCH_CHECK(adds.size() <= 2 && norms.size() <= 2 && norms.size() == hs.size() && !norms.empty(), "residual_norms: at most two adds and norms");
  p.groups = (int)groups;
  p.x = x.data_ptr<float>();
  p.eps = (float)eps;
  p.store = store;
  bool vec = (p.W / groups) % 4 == 0 && aligned16(x);
  const bool f32 = act_f32(hs[0], "h");
  auto act = [&](const Tensor& t, const char* n) {
    same_act(t, hs[0], n);
    vec = vec && aligned16(t) && t.stride(0) % 4 == 0;
  };
  p.R = p.M;
  if (rows.has_value()) {
    TORCH_CHECK(rows->is_cuda() && rows->scalar_type() == at::kLong && rows->is_contiguous() && rows->numel() >= 1 && !store,
                "residual_norms: int64 rows, only read");
    p.R = rows->numel();
    p.rows = rows->data_ptr<int64_t>();
  }
  if (embed.has_value()) {
    act(*embed, "embed");
    TORCH_CHECK(embed->dim() == 2 && embed->is_contiguous() && embed->size(1) == p.W && embed->size(0) >= 1, "residual_norms: embed [V, W]");
    TORCH_CHECK(ids.has_value() && ids->is_cuda() && ids->scalar_type() == at::kLong && ids->is_contiguous() && ids->numel() == p.M,
                "residual_norms: int64 ids [M]");
    p.embed = embed->data_ptr();
    p.ids = ids->data_ptr<int64_t>();
    p.vocab = embed->size(0);
  }
  for (size_t i = 0; i < adds.size(); ++i) {
    act(adds[i], "add");
    TORCH_CHECK(adds[i].dim() == 2 && adds[i].size(0) == p.M && adds[i].size(1) == p.W, "residual_norms: add [M, W]");
    p.add[i] = adds[i].data_ptr();
    p.ld_add[i] = adds[i].stride(0);
  }
  if (pairs.has_value()) {
    act(*pairs, "pairs");
    TORCH_CHECK(pairs->dim() == 2 && pairs->is_contiguous() && pairs->size(1) == p.W && pairs->size(0) >= 1 && pairs->size(0) < (1LL << 31),
                "residual_norms: pairs [P, W]");
    p.pairs = pairs->data_ptr();
    p.npairs = (int)pairs->size(0);
    if (inverse.has_value()) {
      TORCH_CHECK(inverse->dim() == 2 && inverse->size(0) == p.M, "residual_norms: inverse [M, k]");
      p.k = (int)inverse->size(1);
      p.inverse = i32_opt(inverse, p.M * p.k, "inverse");
    } else {   // row m k + j belongs to row m
      TORCH_CHECK(p.npairs % p.M == 0, "residual_norms: as many pairs for every row");
      p.k = (int)(p.npairs / p.M);
    }
  }
  for (size_t i = 0; i < norms.size(); ++i) {
    act(hs[i], "h");
    TORCH_CHECK(hs[i].dim() == 2 && hs[i].size(0) == p.R && hs[i].size(1) == p.W && hs[i].stride(0) == hs[0].stride(0), "residual_norms: h [R, W]");
    p.w[i] = f32_ptr(norms[i], p.W, "norm");
    vec = vec && aligned16(norms[i]);
    p.h[i] = hs[i].data_ptr();
  }
  p.ldh = hs[0].stride(0);
  check_rc(nxd::residual_norms_launch(f32, p, vec, cur_stream()), "residual_norms");
}

// sizes (H, D, rank)
void channel_delta(Tensor proj, int64_t B, int64_t T, std::vector<int64_t> sizes, Tensor w2, Tensor w0, Tensor a_bias, Tensor norm_w,
                   double eps, Tensor pos, Opt lens, Opt slots, Tensor state, Tensor y, double out_scale, int64_t chunk_from) {
  const bool f32 = act_f32(proj, "proj");
  same_act(y, proj, "out");
  same_act(w2, proj, "w2");
  TORCH_CHECK(sizes.size() == 3, "channel_delta: sizes (H, D, rank)");
  nxd::ChannelDeltaParams p{};
  p.B = (int)B;
  p.T = (int)T;
  p.H = (int)sizes[0];
  p.D = (int)sizes[1];
  p.N = (int)sizes[2];
  TORCH_CHECK(B >= 1 && B <= 65535 && T >= 1 && B * T <= (1 << 30), "channel_delta: rows");
  TORCH_CHECK(p.H >= 1 && p.H <= 65535 && p.D >= 1 && p.D <= 256 && p.N >= 1 && p.N <= 4096, "channel_delta: head size up to 256, rank up to 4096");
  p.DP = (p.D + 31) / 32 * 32;
  const int64_t HD = (int64_t)p.H * p.D;
  TORCH_CHECK(proj.dim() == 2 && proj.size(0) == B * T && proj.size(1) >= 5 * HD + p.N, "channel_delta: proj columns");
  TORCH_CHECK(y.dim() == 2 && y.size(0) == B * T && y.size(1) == HD, "channel_delta: out [B T, H D]");
  TORCH_CHECK(w2.dim() == 2 && w2.is_contiguous() && w2.size(0) == HD && w2.size(1) == p.N, "channel_delta: w2 [H D, rank]");
  TORCH_CHECK(state.dim() == 4 && state.is_contiguous() && state.scalar_type() == at::kFloat && state.is_cuda() &&
                  state.size(1) == p.H && state.size(2) == p.D && state.size(3) == p.DP,
              "channel_delta: state fp32 [slots, H, D, D rounded up to 32]");
  TORCH_CHECK(slots.has_value() || B <= state.size(0), "channel_delta: more sequences than slots");
  check_align(state, "state");
  check_align(w2, "w2");
  p.proj = proj.data_ptr();
  p.ldp = proj.stride(0);
  p.w2 = w2.data_ptr();
  p.w0 = f32_ptr(w0, HD, "w0");
  p.a_bias = f32_ptr(a_bias, HD, "a_bias");
  p.norm_w = f32_ptr(norm_w, HD, "norm_w");
  p.eps = (float)eps;
  p.out_scale = (float)out_scale;
  p.pos = pos_ptr(pos, B, &p.pos_stride);
  p.lens = i32_opt(lens, B, "lens");
  p.slots = i32_opt(slots, B, "slots");
  p.nslots = (int)state.size(0);
  p.state = state.data_ptr<float>();
  p.y = y.data_ptr();
  p.ldy = y.stride(0);
  const int C = nxd::channel_delta_chunk(p.DP);
  if (C == 0 || T < chunk_from) {
    check_rc(nxd::channel_delta_step_launch(f32, p, cur_stream()), "channel_delta_step");
    return;
  }
  p.nch = (int)((T + C - 1) / C);
  TORCH_CHECK(p.nch <= 65535, "channel_delta: tokens of one step");
  const int64_t cells = B * p.nch * p.H;
  const int64_t piece = cells * C * p.DP;
  Tensor buf = at::empty({7 * piece + cells * p.DP * (p.DP + 1)}, proj.options().dtype(at::kFloat));
  float* at = buf.data_ptr<float>();
  for (float** q : {&p.cq, &p.co, &p.cw, &p.cy, &p.cb, &p.ck, &p.cv}) *q = at, at += piece;
  p.cs = at;
  p.ce = at + cells * p.DP * p.DP;
  check_rc(nxd::channel_delta_chunk_launch(f32, p, cur_stream()), "channel_delta_chunk");
}

int* i32_new(const Tensor& t, int64_t numel, const char* n) { return const_cast<int*>(i32_opt(t, numel, n)); }

// rule (experts, top, groups, keep): the rule alone
nxd::RouterParams rule_params(const std::vector<int64_t>& rule, double scale, int64_t M) {
  TORCH_CHECK(rule.size() == 4, "router: rule (experts, top, groups, keep)");
  nxd::RouterParams p{};
  p.M = M;
  p.E = (int)rule[0];
  p.top = (int)rule[1];
  p.groups = (int)rule[2];
  p.keep = (int)rule[3];
  TORCH_CHECK(p.M >= 1 && p.E >= 1 && p.E <= 1024, "router: up to 1024 experts");
  TORCH_CHECK(p.groups >= 1 && p.E % p.groups == 0 && p.keep >= 1 && p.keep <= p.groups, "router: equal groups");
  TORCH_CHECK(p.top >= 1 && p.top <= 64 && p.top <= p.keep * (p.E / p.groups) && p.M * p.top < (1LL << 31), "router: up to 64 choices");
  p.scale = (float)scale;
  return p;
}

nxd::RouterParams router_params(const Tensor& logits, const std::vector<int64_t>& rule, double scale) {
  TORCH_CHECK(logits.is_cuda() && logits.dim() == 2 && logits.scalar_type() == at::kFloat && logits.stride(1) == 1, "router: fp32 logits [M, E]");
  auto p = rule_params(rule, scale, logits.size(0));
  TORCH_CHECK(logits.size(1) >= p.E, "router: logits of every expert");
  p.logits = logits.data_ptr<float>();
  p.ldl = logits.stride(0);
  return p;
}

void moe_route(Tensor logits, std::vector<int64_t> rule, double scale, Tensor token, Tensor weight, Tensor inverse, Tensor offs) {
  auto p = router_params(logits, rule, scale);
  const int64_t P = p.M * p.top;
  p.chunks = (int)((p.M + nxd::moe_route_chunk() - 1) / nxd::moe_route_chunk());
  Tensor ints = at::empty({P + (int64_t)p.chunks * p.E}, token.options()), score = at::empty({P}, weight.options());
  p.index = ints.data_ptr<int>();
  p.counts = p.index + P;
  p.score = score.data_ptr<float>();
  p.token = i32_new(token, P, "token");
  p.weight = f32_ptr(weight, P, "weight");
  p.inverse = i32_new(inverse, P, "inverse");
  p.offs = i32_new(offs, p.E + 1, "offs");
  check_rc(nxd::moe_route_launch(p, cur_stream()), "moe_route");
}

void clamped_glu(Tensor gu, double limit, Opt weight, bool sigmoid, Tensor y) {
  const bool f32 = act_f32(gu, "gu");
  same_act(y, gu, "y");
  nxd::GluParams p{};
  p.R = gu.size(0);
  p.F = (int)y.size(1);
  TORCH_CHECK(gu.dim() == 2 && y.dim() == 2 && y.size(0) == p.R && gu.size(1) == 2 * p.F && p.R >= 1 && p.F >= 1, "clamped_glu: gu [R, 2 F], y [R, F]");
  p.gu = gu.data_ptr();
  p.ldg = gu.stride(0);
  p.limit = (float)limit;
  if (weight.has_value()) {
    TORCH_CHECK(weight->is_cuda() && weight->scalar_type() == at::kFloat && weight->dim() == 1 && weight->numel() == p.R, "clamped_glu: fp32 weight [R]");
    p.weight = weight->data_ptr<float>();
    p.ldw = weight->stride(0);
  }
  p.sigmoid = sigmoid;
  p.y = y.data_ptr();
  p.ldy = y.stride(0);
  const bool vec = p.F % 4 == 0 && p.ldg % 4 == 0 && p.ldy % 4 == 0 && aligned16(gu) && aligned16(y);
  check_rc(nxd::clamped_glu_launch(f32, p, vec, cur_stream()), "clamped_glu");
}

void gather_rows(Tensor x, Tensor token, Tensor y) {
  act_f32(x, "x");
  same_act(y, x, "y");
  const int64_t row = x.size(1) * x.element_size(), P = token.numel();
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && y.is_contiguous() && y.size(0) == P && y.size(1) == x.size(1) && row % 16 == 0 && P >= 1,
              "gather_rows: contiguous rows of whole 16-byte pieces");
  check_align(x, "x");
  check_align(y, "y");
  check_rc(nxd::gather_rows_launch(x.data_ptr(), i32_opt(token, P, "token"), y.data_ptr(), x.size(0), P, row, cur_stream()), "gather_rows");
}

// y[rows of e] = x[rows of e] w[e]^T on the matrix cores: bf16, w [E, N, K]
void grouped_linear(Tensor x, Tensor w, Tensor offs, Tensor y) {
  TORCH_CHECK(x.is_cuda() && x.scalar_type() == at::kBFloat16 && w.scalar_type() == at::kBFloat16 && y.scalar_type() == at::kBFloat16, "grouped_linear: bf16");
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && y.dim() == 2 && x.is_contiguous() && w.is_contiguous() && y.is_contiguous(), "grouped_linear: contiguous");
  const int64_t P = x.size(0), E = w.size(0), N = w.size(1), K = w.size(2);
  TORCH_CHECK(x.size(1) == K && y.size(0) == P && y.size(1) == N && K % 8 == 0 && N % 8 == 0, "grouped_linear: shapes");
  TORCH_CHECK(P >= 1 && P < (1LL << 31) && E >= 1 && E < 65536, "grouped_linear: sizes");
  const int* o = i32_opt(offs, E + 1, "offs");
  check_align(x, "x");
  check_align(w, "w");
  check_align(y, "y");
  int rc = nxd::grouped_rowgemm_launch(1, x.data_ptr(), w.data_ptr(), y.data_ptr(), o, (int)E, (int)P, (int)N, (int)K, cur_stream());
  if (rc == -1)
    rc = nxd::grouped_gemm_launch(1, x.data_ptr(), w.data_ptr(), y.data_ptr(), o, (int)E, (int)P, (int)N, (int)K, 0, cur_stream());
  check_rc(rc, "grouped_linear");
}

void expert_rows(Tensor x, Tensor w, Tensor offs, Opt token, Tensor y) {
  const bool f32 = act_f32(x, "x");
  same_act(w, x, "w");
  same_act(y, x, "y");
  nxd::ExpertRowsParams p{};
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && w.is_contiguous() && y.dim() == 2 && y.is_contiguous(), "expert_rows: contiguous w and y");
  p.E = (int)w.size(0);
  p.N = (int)w.size(1);
  p.K = (int)w.size(2);
  p.P = y.size(0);
  TORCH_CHECK(x.size(1) == p.K && y.size(1) == p.N && p.P >= 1 && p.K <= 40960, "expert_rows: shapes");
  TORCH_CHECK(token.has_value() || x.size(0) == p.P, "expert_rows: a row of x for each row of y");
  p.x = x.data_ptr();
  p.ldx = x.stride(0);
  p.nx = x.size(0);
  p.token = i32_opt(token, p.P, "token");
  p.w = w.data_ptr();
  p.offs = i32_opt(offs, p.E + 1, "offs");
  p.y = y.data_ptr();
  check_rc(nxd::expert_rows_launch(f32, p, cur_stream()), "expert_rows");
}

// y [M (top + shared), W]: outputs of a token's experts, weighted, then its shared expert's
void experts_few(Tensor h, Tensor router, std::vector<int64_t> rule, double scale, Tensor up, Tensor down, double limit, Opt sup,
                 Opt sdown, double slimit, Opt gate, Tensor y) {
  auto bf = [](const Tensor& t, int64_t d, const char* n) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kBFloat16 && t.dim() == d && t.is_contiguous(), "experts_few: ", n, ": contiguous bf16");
    check_align(t, n);
    return static_cast<uint16_t*>(t.data_ptr());
  };
  nxd::ExpertFewParams p{};
  p.h = bf(h, 2, "h");
  const auto r = rule_params(rule, scale, h.size(0));
  p.M = (int)h.size(0);
  p.W = (int)h.size(1);
  p.ldh = h.stride(0);
  p.E = r.E;
  p.top = r.top;
  p.router = bf(router, 2, "router");
  p.up = bf(up, 3, "up");
  p.down = bf(down, 3, "down");
  p.F = (int)down.size(2);
  p.shared = sup.has_value() ? 1 : 0;
  TORCH_CHECK(sup.has_value() == sdown.has_value(), "experts_few: both matrices of the shared expert");
  if (p.shared) {
    p.sup = bf(*sup, 2, "shared up");
    p.sdown = bf(*sdown, 2, "shared down");
    p.FS = (int)sdown->size(1);
    TORCH_CHECK(sup->size(0) == 2 * p.FS && sup->size(1) == p.W && sdown->size(0) == p.W, "experts_few: shared expert's shapes");
  }
  TORCH_CHECK(p.M <= 64 && p.W % 8 == 0 && p.F % 8 == 0 && p.FS % 8 == 0 && p.F >= 8 && p.W >= 8 && p.W < (1 << 24) && (int64_t)p.M * p.top * p.F < (1LL << 31) && p.FS < (1 << 24), "experts_few: up to 64 tokens, sizes multiples of 8");
  TORCH_CHECK(!(p.shared && gate.has_value()) && (!p.shared || p.M <= 16), "experts_few: the shared expert here (up to 16 tokens), or its gate");
  p.gate = f32_opt(gate, p.M, "gate");
  TORCH_CHECK(router.size(0) >= p.E + (p.shared || p.gate ? 1 : 0) && router.size(1) == p.W, "experts_few: router [>= E + shared, W]");
  TORCH_CHECK(up.size(0) == p.E && up.size(1) == 2 * p.F && up.size(2) == p.W && down.size(0) == p.E && down.size(1) == p.W, "experts_few: experts' shapes");
  const int64_t slots = p.top + p.shared;
  p.y = bf(y, 2, "y");
  TORCH_CHECK(y.size(0) == p.M * slots && y.size(1) == p.W, "experts_few: y [M (top + shared), W]");
  p.limit = (float)limit;
  p.slimit = (float)slimit;
  Tensor index = at::empty({p.M, p.top}, h.options().dtype(at::kInt)), score = at::empty({p.M, slots}, h.options().dtype(at::kFloat));
  Tensor a = at::empty({(int64_t)p.M * p.top * p.F + (int64_t)p.M * p.FS}, h.options());
  p.index = index.data_ptr<int>();
  p.score = score.data_ptr<float>();
  p.a = static_cast<uint16_t*>(a.data_ptr());
  p.sa = p.a + (int64_t)p.M * p.top * p.F;
  check_rc(nxd::experts_few_launch(r, p, cur_stream()), "experts_few");
}

// y [M, N] = x [M, K] w^T, up to 16 rows
void linear_few(Tensor x, Tensor w, Tensor y) {
  for (const Tensor* t : {&x, &w, &y})
    TORCH_CHECK(t->is_cuda() && t->scalar_type() == at::kBFloat16 && t->dim() == 2 && t->stride(1) == 1, "linear_few: bf16 matrices");
  nxd::LinearFewParams p{};
  p.M = (int)x.size(0);
  p.K = (int)x.size(1);
  p.N = (int)w.size(0);
  TORCH_CHECK(p.M >= 1 && p.M <= 16 && p.K >= 8 && p.K % 8 == 0 && p.N >= 1 && x.stride(0) < (1 << 24), "linear_few: 1..16 rows, K a multiple of 8");
  TORCH_CHECK(w.is_contiguous() && w.size(1) == p.K && y.size(0) == p.M && y.size(1) == p.N && x.stride(0) % 8 == 0, "linear_few: shapes");
  check_align(x, "x");
  check_align(w, "w");
  check_align(y, "y");
  p.x = static_cast<const uint16_t*>(x.data_ptr());
  p.ldx = x.stride(0);
  p.w = static_cast<const uint16_t*>(w.data_ptr());
  p.y = static_cast<uint16_t*>(y.data_ptr());
  p.ldy = y.stride(0);
  check_rc(nxd::linear_few_launch(p, cur_stream()), "linear_few");
}

}  // namespace

void register_parallel(pybind11::module& m) {
  m.def("residual_norms", &residual_norms);
  m.def("channel_delta", &channel_delta);
  m.def("moe_route", &moe_route);
  m.def("clamped_glu", &clamped_glu);
  m.def("gather_rows", &gather_rows);
  m.def("grouped_linear", &grouped_linear);
  m.def("expert_rows", &expert_rows);
  m.def("experts_few", &experts_few);
  m.def("linear_few", &linear_few);
}
