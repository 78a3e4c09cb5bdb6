// Python bindings of the hybrid-decoder kernels (module `neuronx_distributed_llama3_2_amd._hybrid`).
// Every entry point checks shapes, types and the kernels' size limits on the host before it launches
// on the caller's current stream.
#include "bindings_util.h"
#include "delta_rule.h"
#include "gemv_hyper.h"
#include "window_attn.h"

void register_gemm(pybind11::module& m);      // ../gemm.cpp
void register_parallel(pybind11::module& m);  // bindings_parallel.cpp

namespace nxd {
int hyper_step_launch(bool, float*, const void*, const int64_t*, int64_t, const void*, int64_t, const float*, const float*,
                      const float*, const float*, const float*, float, void*, int64_t, const int64_t*, bool, int64_t, int,
                      int, hipStream_t);
int relu_squared_launch(bool, const void*, void*, int64_t, hipStream_t);
int softcap_launch(float*, int64_t, float, hipStream_t);
int delta_prep_launch(bool, const DeltaParams&, hipStream_t);
int delta_scan_launch(bool, const DeltaParams&, hipStream_t);
int delta_chunk_launch(bool, const DeltaParams&, hipStream_t);
int delta_out_launch(bool, const DeltaParams&, hipStream_t);
int delta_decode_launch(bool, const DeltaParams&, hipStream_t);
int attn_prep_launch(bool, const WindowAttnParams&, hipStream_t);
bool attn_prompt_supported(const WindowAttnParams&);
int attn_prompt_launch(const WindowAttnParams&, hipStream_t);
int attn_row_launch(bool, const WindowAttnParams&, hipStream_t);
void attn_decode_plan(WindowAttnParams&, int64_t);
int attn_decode_launch(bool, const WindowAttnParams&, hipStream_t);
int gemv_hyper_launch(int, const GemvHyperParams&, hipStream_t);
int pooled_prep_launch(bool, const WindowAttnParams&, hipStream_t);
}  // namespace nxd

namespace {

using namespace nxd::bind;

void hyper_step(Tensor x, Opt embed, Opt ids, Opt y, Opt bias, Opt mix, Opt write, Opt read, Opt norm_w, double eps, Opt h,
                Opt rows, bool store) {
  TORCH_CHECK(x.dim() == 3 && x.is_cuda() && x.scalar_type() == at::kFloat && x.is_contiguous(), "hyper_step: x fp32 [M, S, W]");
  const int64_t M = x.size(0), S = x.size(1), W = x.size(2);
  TORCH_CHECK(S >= 1 && S <= 8, "hyper_step: 1..8 streams");
  TORCH_CHECK(W >= 1 && W <= 16384, "hyper_step: width up to 16384");
  TORCH_CHECK(h.has_value() == read.has_value() && h.has_value() == norm_w.has_value(), "hyper_step: read, norm and h together");
  TORCH_CHECK(h.has_value() || y.has_value(), "hyper_step: nothing to do");
  check_align(x, "x");
  bool f32 = false, have = false;
  auto act = [&](const Tensor& t, const char* n) {
    const bool f = act_f32(t, n);
    TORCH_CHECK(!have || f == f32, "hyper_step: activation types differ");
    f32 = f;
    have = true;
    check_align(t, n);
  };
  const int64_t R = rows.has_value() ? rows->numel() : M;
  if (rows.has_value()) {
    TORCH_CHECK(rows->is_cuda() && rows->scalar_type() == at::kLong && rows->is_contiguous(), "hyper_step: int64 rows");
    TORCH_CHECK(!store, "hyper_step: selected rows are only read");
  }
  if (embed.has_value()) {
    act(*embed, "embed");
    TORCH_CHECK(embed->is_contiguous() && embed->dim() == 2 && embed->size(1) == W, "hyper_step: embed [V, W]");
    TORCH_CHECK(ids.has_value() && ids->is_cuda() && ids->scalar_type() == at::kLong && ids->is_contiguous() && ids->numel() == M,
                "hyper_step: int64 ids [M]");
  }
  int64_t ldy = 0, ldh = 0;
  if (y.has_value()) {
    act(*y, "y");
    TORCH_CHECK(y->dim() == 2 && y->size(0) == M && y->size(1) == W, "hyper_step: y [M, W]");
    TORCH_CHECK(mix.has_value() && write.has_value(), "hyper_step: mix and write with y");
    ldy = y->stride(0);
  }
  if (h.has_value()) {
    act(*h, "h");
    TORCH_CHECK(h->dim() == 2 && h->size(0) == R && h->size(1) == W, "hyper_step: h [R, W]");
    ldh = h->stride(0);
  }
  check_rc(nxd::hyper_step_launch(f32, x.data_ptr<float>(), embed.has_value() ? embed->data_ptr() : nullptr,
                                  embed.has_value() ? ids->data_ptr<int64_t>() : nullptr,
                                  embed.has_value() ? embed->size(0) : 0, y.has_value() ? y->data_ptr() : nullptr, ldy,
                                  f32_opt(bias, W, "bias"), f32_opt(mix, S * S, "mix"), f32_opt(write, S, "write"),
                                  f32_opt(read, S, "read"), f32_opt(norm_w, W, "norm_w"), (float)eps,
                                  h.has_value() ? h->data_ptr() : nullptr, ldh,
                                  rows.has_value() ? rows->data_ptr<int64_t>() : nullptr, store, R, (int)S, (int)W,
                                  cur_stream()),
           "hyper_step");
}

void relu_squared(Tensor x, Tensor y) {
  const bool f32 = act_f32(x, "x");
  same_act(y, x, "y");
  TORCH_CHECK(x.is_contiguous() && y.is_contiguous() && x.numel() == y.numel(), "relu_squared: contiguous, equal sizes");
  check_align(x, "x");
  check_align(y, "y");
  check_rc(nxd::relu_squared_launch(f32, x.data_ptr(), y.data_ptr(), x.numel(), cur_stream()), "relu_squared");
}

void softcap_(Tensor x, double cap) {
  TORCH_CHECK(x.is_cuda() && x.scalar_type() == at::kFloat && x.is_contiguous() && cap > 0, "softcap_: contiguous fp32, cap > 0");
  check_rc(nxd::softcap_launch(x.data_ptr<float>(), x.numel(), (float)cap, cur_stream()), "softcap_");
}

// The recurrence over T new tokens of B sequences.  one launch (T == 1 and `fused`) or three with the
// fp32 intermediates; sizes (H, G, D, V).
void delta_rule(Tensor proj, int64_t B, int64_t T, std::vector<int64_t> sizes, Tensor conv, Tensor a_log, Tensor dt_bias,
                Tensor norm_w, double eps, Tensor pos, Opt lens, Opt slots, Tensor state, Tensor ring, Tensor y, bool fused,
                int64_t chunk_from) {
  const bool f32 = act_f32(proj, "proj");
  same_act(ring, proj, "ring");
  same_act(y, proj, "y");
  TORCH_CHECK(sizes.size() == 4, "delta_rule: sizes (H, G, D, V)");
  nxd::DeltaParams p{};
  p.B = (int)B;
  p.T = (int)T;
  p.H = (int)sizes[0];
  p.G = (int)sizes[1];
  p.D = (int)sizes[2];
  p.V = (int)sizes[3];
  TORCH_CHECK(B >= 1 && T >= 1 && B * T <= (1 << 30), "delta_rule: rows");
  TORCH_CHECK(p.G >= 1 && p.H >= 1 && p.H % p.G == 0 && p.H <= 65535 && B <= 65535, "delta_rule: head layout");
  TORCH_CHECK(p.D >= 1 && p.D <= 256 && p.V >= 1 && p.V <= 256, "delta_rule: head sizes up to 256");
  p.DP = (p.D + 31) / 32 * 32;
  p.C = 2 * p.G * p.D + p.H * p.V;
  TORCH_CHECK(conv.dim() == 2 && conv.size(1) == p.C && conv.size(0) >= 1, "delta_rule: conv [taps, C]");
  p.taps = (int)conv.size(0);
  TORCH_CHECK(proj.dim() == 2 && proj.size(0) == B * T && proj.size(1) >= p.C + p.H * p.V + 2 * p.H, "delta_rule: proj columns");
  TORCH_CHECK(y.dim() == 2 && y.size(0) == B * T && y.size(1) == p.H * p.V, "delta_rule: y [B T, H V]");
  TORCH_CHECK(state.dim() == 4 && state.is_contiguous() && state.scalar_type() == at::kFloat && state.is_cuda() &&
                  state.size(1) == p.H && state.size(2) == p.V && state.size(3) == p.DP,
              "delta_rule: state fp32 [slots, H, V, D rounded up to 32]");
  const int64_t ns = state.size(0);
  TORCH_CHECK(ring.is_contiguous() && ring.dim() == 3 && ring.size(0) == ns && ring.size(1) == p.taps && ring.size(2) == p.C,
              "delta_rule: ring [slots, taps, C]");
  TORCH_CHECK(slots.has_value() || B <= ns, "delta_rule: more sequences than slots");
  check_align(state, "state");
  p.proj = proj.data_ptr();
  p.ldp = proj.stride(0);
  p.conv = f32_ptr(conv, (int64_t)p.taps * p.C, "conv");
  p.a_log = f32_ptr(a_log, p.H, "a_log");
  p.dt_bias = f32_ptr(dt_bias, p.H, "dt_bias");
  p.norm_w = f32_ptr(norm_w, p.V, "norm_w");
  p.qscale = (float)(1.0 / std::sqrt((double)p.D));
  p.eps = (float)eps;
  p.pos = pos_ptr(pos, B, &p.pos_stride);
  p.lens = i32_opt(lens, B, "lens");
  p.slots = i32_opt(slots, B, "slots");
  p.nslots = (int)ns;
  p.state = state.data_ptr<float>();
  p.ring = ring.data_ptr();
  p.y = y.data_ptr();
  p.ldy = y.stride(0);
  if (fused && T == 1 && !lens.has_value()) {
    check_rc(nxd::delta_decode_launch(f32, p, cur_stream()), "delta_decode");
    return;
  }
  auto opt = proj.options().dtype(at::kFloat);
  const int64_t M = B * T;
  if (T >= chunk_from) p.nch = (int)((T + 63) / 64);
  TORCH_CHECK(p.nch <= 65535, "delta_rule: tokens of one step");
  const int64_t Mq = p.nch > 0 ? B * p.nch * 64 : M;   // whole chunks of q and k
  Tensor qk = at::empty({2, Mq, p.G, p.DP}, opt), vo = at::empty({2, M, p.H, p.V}, opt), gb = at::empty({2, M, p.H}, opt);
  p.qn = qk.data_ptr<float>();
  p.kn = p.qn + Mq * p.G * p.DP;
  p.vn = vo.data_ptr<float>();
  p.o = p.vn + M * p.H * p.V;
  p.lg = gb.data_ptr<float>();
  p.beta = p.lg + M * p.H;
  check_rc(nxd::delta_prep_launch(f32, p, cur_stream()), "delta_prep");
  Tensor cells;   // (outlives the launches below)
  if (p.nch > 0) {
    const int64_t n = B * p.nch * p.H;
    cells = at::empty({n * 64 * (p.DP + (p.V + 15) / 16 * 16 + 64 + 2)}, opt);
    p.cw = cells.data_ptr<float>();
    p.cp = p.cw + n * 64 * p.DP;
    p.ceg = p.cp + n * 64 * 64;
    p.cy = p.ceg + n * 64 * 2;
    check_rc(nxd::delta_chunk_launch(f32, p, cur_stream()), "delta_chunk");
  } else {
    check_rc(nxd::delta_scan_launch(f32, p, cur_stream()), "delta_scan");
  }
  check_rc(nxd::delta_out_launch(f32, p, cur_stream()), "delta_out");
}

// sizes (H, G, maps, D, V)
nxd::WindowAttnParams attn_params(const Tensor& buf, int64_t B, int64_t T, const std::vector<int64_t>& sizes,
                                  const Tensor& pos, const Opt& lens, const Opt& slots, const Tensor& kc, const Tensor& vc) {
  act_f32(buf, "buf");
  same_act(kc, buf, "k cache");
  same_act(vc, buf, "v cache");
  TORCH_CHECK(sizes.size() == 5, "attention: sizes (H, G, maps, D, V)");
  nxd::WindowAttnParams p{};
  p.B = (int)B;
  p.T = (int)T;
  p.H = (int)sizes[0];
  p.G = (int)sizes[1];
  p.maps = (int)sizes[2];
  p.D = (int)sizes[3];
  p.V = (int)sizes[4];
  TORCH_CHECK(B >= 1 && T >= 1 && B * T <= (1 << 30), "attention: rows");
  TORCH_CHECK(p.G >= 1 && p.H % p.G == 0 && p.H >= 1 && (p.maps == 1 || p.maps == 2), "attention: head layout");
  TORCH_CHECK(p.D >= 2 && p.D <= 256 && p.V >= 1 && p.V <= 256, "attention: head sizes up to 256");
  TORCH_CHECK(buf.dim() == 2 && buf.size(0) == B * T && buf.size(1) >= (p.H + p.G) * p.maps * p.D + p.G * p.V,
              "attention: projection columns");
  TORCH_CHECK(kc.dim() == 4 && kc.is_contiguous() && kc.size(1) == p.G * p.maps && kc.size(3) == p.D,
              "attention: k cache [slots, G maps, cap, D]");
  TORCH_CHECK(vc.dim() == 4 && vc.is_contiguous() && vc.size(0) == kc.size(0) && vc.size(1) == p.G && vc.size(2) == kc.size(2) &&
                  vc.size(3) == p.V,
              "attention: v cache [slots, G, cap, V]");
  TORCH_CHECK(kc.size(2) >= 1 && kc.size(2) < (1 << 30), "attention: cache length");
  TORCH_CHECK(slots.has_value() || B <= kc.size(0), "attention: more sequences than slots");
  p.buf = buf.data_ptr();
  p.ldb = buf.stride(0);
  p.pos = pos_ptr(pos, B, &p.pos_stride);
  p.lens = i32_opt(lens, B, "lens");
  p.slots = i32_opt(slots, B, "slots");
  p.nslots = (int)kc.size(0);
  p.kc = kc.data_ptr();
  p.vc = vc.data_ptr();
  p.cap = (int)kc.size(2);
  p.v_off = (p.H + p.G) * p.maps * p.D;
  p.kbuf = static_cast<const char*>(p.buf) + (int64_t)p.H * p.maps * p.D * buf.element_size();
  p.vbuf = static_cast<const char*>(p.buf) + (int64_t)p.v_off * buf.element_size();
  p.ldk = p.ldv = p.ldb;
  return p;
}

void set_prep(nxd::WindowAttnParams& p, const Opt& bias, const Opt& qn_w, const Opt& kn_w, double eps, const Tensor& cos_t,
              const Tensor& sin_t) {
  p.bias = f32_opt(bias, (p.H + p.G) * p.maps * p.D + p.G * p.V, "bias");
  TORCH_CHECK(qn_w.has_value() == kn_w.has_value(), "attention: both head norms or none");
  p.qn_w = f32_opt(qn_w, p.D, "qn_w");
  p.kn_w = f32_opt(kn_w, p.D, "kn_w");
  p.eps = (float)eps;
  TORCH_CHECK(cos_t.dim() == 2 && cos_t.sizes() == sin_t.sizes() && cos_t.size(0) >= 1 && 2 * cos_t.size(1) <= p.D,
              "attention: cos / sin [positions, rotated pairs]");
  p.cos_t = f32_ptr(cos_t, cos_t.numel(), "cos");
  p.sin_t = f32_ptr(sin_t, sin_t.numel(), "sin");
  p.rot = 2 * (int)cos_t.size(1);
  p.max_pos = (int)cos_t.size(0);
}

void set_rule(nxd::WindowAttnParams& p, double scale, double softcap, int64_t window, double lam, double out_scale,
              double out_eps, const Tensor& buf, const Tensor& y) {
  same_act(y, buf, "y");
  TORCH_CHECK(y.dim() == 2 && y.size(0) == (int64_t)p.B * p.T && y.size(1) == p.H * p.V, "attention: y [B T, H V]");
  p.scale = (float)scale;
  p.softcap = (float)softcap;
  p.window = window > 0 && window < (1 << 30) ? (int)window : 0;
  p.lam = (float)lam;
  p.out_scale = (float)out_scale;
  p.out_eps = (float)out_eps;
  p.y = y.data_ptr();
  p.ldy = y.stride(0);
}

void attn_prep(Tensor buf, int64_t B, int64_t T, std::vector<int64_t> sizes, Opt bias, Opt qn_w, Opt kn_w, double eps,
               Tensor cos_t, Tensor sin_t, Tensor pos, Opt lens, Opt slots, Tensor kc, Tensor vc) {
  auto p = attn_params(buf, B, T, sizes, pos, lens, slots, kc, vc);
  set_prep(p, bias, qn_w, kn_w, eps, cos_t, sin_t);
  check_rc(nxd::attn_prep_launch(buf.scalar_type() == at::kFloat, p, cur_stream()), "attn_prep");
}

// from_buf: the new tokens start at position 0 and see only each other
void window_attn(Tensor buf, int64_t B, int64_t T, std::vector<int64_t> sizes, double scale, double softcap, int64_t window,
                 double lam, double out_scale, double out_eps, Tensor pos, Opt lens, Opt slots, Tensor kc, Tensor vc, Tensor y,
                 bool from_buf, bool fused) {
  auto p = attn_params(buf, B, T, sizes, pos, lens, slots, kc, vc);
  set_rule(p, scale, softcap, window, lam, out_scale, out_eps, buf, y);
  TORCH_CHECK(from_buf || T <= p.cap, "window_attn: ", T, " new tokens do not fit a ring of ", p.cap);
  p.from_buf = from_buf ? 1 : 0;
  const bool f32 = buf.scalar_type() == at::kFloat;
  if (fused && !f32 && nxd::attn_prompt_supported(p)) {
    check_rc(nxd::attn_prompt_launch(p, cur_stream()), "attn_prompt");
    return;
  }
  check_rc(nxd::attn_row_launch(f32, p, cur_stream()), "window_attn");
}

// one new token per sequence: preparation, cache write and attention.  tickets: int32, zero, at least B H
void attn_decode(Tensor buf, std::vector<int64_t> sizes, Opt bias, Opt qn_w, Opt kn_w, double eps, Tensor cos_t, Tensor sin_t,
                 double scale, double softcap, int64_t window, double lam, double out_scale, double out_eps, Tensor pos,
                 Opt slots, Tensor kc, Tensor vc, Tensor tickets, Tensor y) {
  const int64_t B = buf.size(0);
  auto p = attn_params(buf, B, 1, sizes, pos, Opt(), slots, kc, vc);
  set_prep(p, bias, qn_w, kn_w, eps, cos_t, sin_t);
  set_rule(p, scale, softcap, window, lam, out_scale, out_eps, buf, y);
  TORCH_CHECK(p.H <= 65535 && B <= 65535, "attn_decode: grid");
  const int64_t seen = p.window > 0 ? std::min<int64_t>(p.window, p.cap) : p.cap;
  nxd::attn_decode_plan(p, seen);
  TORCH_CHECK(tickets.is_cuda() && tickets.scalar_type() == at::kInt && tickets.is_contiguous() && tickets.numel() >= B * p.H,
              "attn_decode: int32 tickets, B H of them");
  Tensor part;
  if (p.splits > 1) {
    part = at::empty({B * p.H * p.splits * p.maps * (p.V + 2)}, buf.options().dtype(at::kFloat));
    p.part = part.data_ptr<float>();
    p.tickets = tickets.data_ptr<int>();
  }
  check_rc(nxd::attn_decode_launch(buf.scalar_type() == at::kFloat, p, cur_stream()), "attn_decode");
}

// Pooled blocks.  sizes (H, G, D); buf columns q (H D) | k (G D, also the values); kn [B T, G D] normalised keys
nxd::WindowAttnParams pooled_params(const Tensor& buf, const Opt& kn, int64_t B, int64_t T, const std::vector<int64_t>& sizes,
                                    int64_t window, int64_t pool, const Tensor& pos, const Opt& lens, const Opt& slots,
                                    const Tensor& kc, const Tensor& vc, const Tensor& pk, const Tensor& pv) {
  const bool f32 = act_f32(buf, "buf");
  same_act(kc, buf, "k cache");
  same_act(vc, buf, "v cache");
  same_act(pk, buf, "pooled k");
  same_act(pv, buf, "pooled v");
  TORCH_CHECK(sizes.size() == 3, "pooled attention: sizes (H, G, D)");
  nxd::WindowAttnParams p{};
  p.B = (int)B;
  p.T = (int)T;
  p.H = (int)sizes[0];
  p.G = (int)sizes[1];
  p.maps = 1;
  p.D = p.V = (int)sizes[2];
  TORCH_CHECK(B >= 1 && B <= 65535 && T >= 1 && B * T <= (1 << 30), "pooled attention: rows");
  TORCH_CHECK(p.G >= 1 && p.H >= 1 && p.H <= 65535 && p.H % p.G == 0 && p.D >= 2 && p.D <= 256, "pooled attention: head layout, size up to 256");
  TORCH_CHECK(buf.dim() == 2 && buf.size(0) == B * T && buf.size(1) >= (p.H + p.G) * p.D, "pooled attention: projection columns");
  TORCH_CHECK(kc.dim() == 4 && kc.is_contiguous() && kc.size(1) == p.G && kc.size(3) == p.D && vc.is_contiguous() && vc.sizes() == kc.sizes(),
              "pooled attention: caches [slots, G, cap, D]");
  TORCH_CHECK(pk.dim() == 4 && pk.is_contiguous() && pk.size(0) == kc.size(0) && pk.size(1) == p.G && pk.size(3) == p.D &&
                  pv.is_contiguous() && pv.sizes() == pk.sizes() && pk.size(2) >= 1 && pk.size(2) < (1 << 30),
              "pooled attention: pooled caches [slots, G, blocks, D]");
  TORCH_CHECK(kc.size(2) >= 1 && kc.size(2) < (1 << 30), "pooled attention: cache length");
  TORCH_CHECK(slots.has_value() || B <= kc.size(0), "pooled attention: more sequences than slots");
  TORCH_CHECK(window >= 1 && window < (1 << 30) && pool >= 1 && pool < (1 << 30), "pooled attention: window and block");
  for (const Tensor* t : {&kc, &vc, &pk, &pv}) check_align(*t, "caches");
  p.buf = buf.data_ptr();
  p.ldb = buf.stride(0);
  p.v_off = p.H * p.D;
  p.vbuf = static_cast<const char*>(p.buf) + (int64_t)p.v_off * buf.element_size();
  p.ldv = p.ldb;
  if (kn.has_value()) {
    same_act(*kn, buf, "kn");
    TORCH_CHECK(kn->dim() == 2 && kn->size(0) == B * T && kn->size(1) == p.G * p.D, "pooled attention: kn [B T, G D]");
    p.kbuf = kn->data_ptr();
    p.ldk = kn->stride(0);
  }
  p.pos = pos_ptr(pos, B, &p.pos_stride);
  p.lens = i32_opt(lens, B, "lens");
  p.slots = i32_opt(slots, B, "slots");
  p.nslots = (int)kc.size(0);
  p.kc = kc.data_ptr();
  p.vc = vc.data_ptr();
  p.cap = (int)kc.size(2);
  p.window = (int)window;
  p.pool = (int)pool;
  p.pcap = (int)pk.size(2);
  p.pk = pk.data_ptr();
  p.pv = pv.data_ptr();
  p.norm_all = true;
  (void)f32;
  return p;
}

void set_pooled_norms(nxd::WindowAttnParams& p, const Tensor& qn_w, const Tensor& kn_w, double eps) {
  p.qn_w = f32_ptr(qn_w, p.H * p.D, "q norm");
  p.kn_w = f32_ptr(kn_w, p.G * p.D, "k norm");
  check_align(qn_w, "q norm");
  check_align(kn_w, "k norm");
  p.eps = (float)eps;
}

void set_pooled_out(nxd::WindowAttnParams& p, double scale, const Tensor& buf, const Tensor& out, double out_scale) {
  same_act(out, buf, "out");
  TORCH_CHECK(out.dim() == 2 && out.size(0) == (int64_t)p.B * p.T && out.size(1) == p.H * p.D, "pooled attention: out [B T, H D]");
  p.scale = (float)scale;
  p.out_scale = (float)out_scale;
  p.y = out.data_ptr();
  p.ldy = out.stride(0);
}

void check_ring(const nxd::WindowAttnParams& p, bool prompt) {
  // a ring that wraps must still hold what the first new token sees and the blocks the step completes
  TORCH_CHECK(prompt || p.T <= p.cap, "pooled attention: ", p.T, " new tokens do not fit a ring of ", p.cap);
}

void pooled_prep(Tensor buf, Tensor kn, int64_t B, int64_t T, std::vector<int64_t> sizes, Tensor qn_w, Tensor kn_w, double eps,
                 int64_t pool, Tensor pos, Opt lens, Opt slots, Tensor kc, Tensor vc, Tensor pk, Tensor pv, bool prompt) {
  auto p = pooled_params(buf, kn, B, T, sizes, 1, pool, pos, lens, slots, kc, vc, pk, pv);
  check_ring(p, prompt);
  set_pooled_norms(p, qn_w, kn_w, eps);
  p.from_buf = prompt ? 1 : 0;
  check_rc(nxd::pooled_prep_launch(buf.scalar_type() == at::kFloat, p, cur_stream()), "pooled_prep");
}

void pooled_attn(Tensor buf, Tensor kn, int64_t B, int64_t T, std::vector<int64_t> sizes, double scale, int64_t window, int64_t pool,
                 Tensor pos, Opt lens, Opt slots, Tensor kc, Tensor vc, Tensor pk, Tensor pv, Tensor out, double out_scale,
                 bool prompt, bool fused) {
  auto p = pooled_params(buf, kn, B, T, sizes, window, pool, pos, lens, slots, kc, vc, pk, pv);
  check_ring(p, prompt);
  set_pooled_out(p, scale, buf, out, out_scale);
  p.from_buf = prompt ? 1 : 0;
  const bool f32 = buf.scalar_type() == at::kFloat;
  if (fused && !f32 && nxd::attn_prompt_supported(p)) {
    check_rc(nxd::attn_prompt_launch(p, cur_stream()), "attn_prompt");
    return;
  }
  check_rc(nxd::attn_row_launch(f32, p, cur_stream()), "pooled_attn");
}

void pooled_decode(Tensor buf, std::vector<int64_t> sizes, Tensor qn_w, Tensor kn_w, double eps, double scale, int64_t window,
                   int64_t pool, Tensor pos, Opt slots, Tensor kc, Tensor vc, Tensor pk, Tensor pv, Tensor tickets, Tensor out,
                   double out_scale) {
  const int64_t B = buf.size(0);
  auto p = pooled_params(buf, Opt(), B, 1, sizes, window, pool, pos, Opt(), slots, kc, vc, pk, pv);
  set_pooled_norms(p, qn_w, kn_w, eps);
  set_pooled_out(p, scale, buf, out, out_scale);
  p.max_pos = 1 << 30;
  nxd::attn_decode_plan(p, std::min(p.window, p.cap) + p.pcap);
  TORCH_CHECK(tickets.is_cuda() && tickets.scalar_type() == at::kInt && tickets.is_contiguous() && tickets.numel() >= B * p.H,
              "pooled_decode: int32 tickets, B H of them");
  Tensor part;
  if (p.splits > 1) {
    part = at::empty({B * p.H * p.splits * (p.V + 2)}, buf.options().dtype(at::kFloat));
    p.part = part.data_ptr<float>();
    p.tickets = tickets.data_ptr<int>();
  }
  check_rc(nxd::attn_decode_launch(buf.scalar_type() == at::kFloat, p, cur_stream()), "pooled_decode");
}

// y = epi(x w^T), 1..4 rows of bf16; x bf16 [M, K], or u fp32 [M, K] normalised on the way in.  epi: 0 bf16,
// 1 squared ReLU, 2 fp32 with cap, 3 into the streams (y unused, `un` receives the next sublayer's input)
void gemv_hyper(int64_t epi, Opt x, Opt u, Opt norm_w, double eps, Tensor w, Opt y, double cap, Opt streams, Opt bias, Opt mix,
                Opt write, Opt read, Opt un, double alpha) {
  nxd::GemvHyperParams p{};
  TORCH_CHECK(epi >= 0 && epi <= 3, "gemv_hyper: epi 0..3");
  TORCH_CHECK(x.has_value() != u.has_value() && u.has_value() == norm_w.has_value(), "gemv_hyper: x, or u with norm_w");
  TORCH_CHECK(w.is_cuda() && w.dim() == 2 && w.scalar_type() == at::kBFloat16 && w.stride(1) == 1 && w.stride(0) % 8 == 0,
              "gemv_hyper: w bf16 [N, K]");
  const Tensor& in = x.has_value() ? *x : *u;
  TORCH_CHECK(in.is_cuda() && in.dim() == 2 && in.size(1) == w.size(1) && in.stride(1) == 1, "gemv_hyper: input [M, K]");
  const int64_t M = in.size(0), N = w.size(0), K = w.size(1);
  TORCH_CHECK(M >= 1 && M <= 4 && N >= 1 && K >= 8 && K % 8 == 0, "gemv_hyper: 1..4 rows, K a multiple of 8");
  check_align(in, "input");
  check_align(w, "w");
  p.M = (int)M;
  p.N = (int)N;
  p.K = (int)K;
  p.w = static_cast<const uint16_t*>(w.data_ptr());
  p.ldw = w.stride(0);
  p.eps = (float)eps;
  p.cap = (float)cap;
  p.alpha = (float)alpha;
  if (x.has_value()) {
    TORCH_CHECK(x->scalar_type() == at::kBFloat16 && x->stride(0) % 8 == 0, "gemv_hyper: x bf16, rows 16-byte aligned");
    p.x = static_cast<const uint16_t*>(x->data_ptr());
    p.ldx = x->stride(0);
  } else {
    p.u = f32_ptr(*u, M * K, "u");
    p.norm_w = f32_ptr(*norm_w, K, "norm_w");
    check_align(*norm_w, "norm_w");
    TORCH_CHECK(M * K <= 24576, "gemv_hyper: normalised rows must fit 48 KB of LDS");
  }
  if (epi == 3) {
    TORCH_CHECK(x.has_value() && streams.has_value() && mix.has_value() && write.has_value() && read.has_value() && un.has_value(),
                "gemv_hyper: streams, mix, write, read, un");
    TORCH_CHECK(streams->dim() == 3 && streams->size(0) == M && streams->size(2) == N && streams->size(1) >= 1 && streams->size(1) <= 8,
                "gemv_hyper: streams [M, S, N]");
    p.S = (int)streams->size(1);
    p.streams = f32_ptr(*streams, M * p.S * N, "streams");
    p.bias = f32_opt(bias, N, "bias");
    p.mix = f32_ptr(*mix, p.S * p.S, "mix");
    p.write = f32_ptr(*write, p.S, "write");
    p.read = f32_ptr(*read, p.S, "read");
    p.un = f32_ptr(*un, M * N, "un");
  } else {
    TORCH_CHECK(y.has_value() && y->is_cuda() && y->dim() == 2 && y->size(0) == M && y->size(1) == N && y->stride(1) == 1 &&
                    y->scalar_type() == (epi == 2 ? at::kFloat : at::kBFloat16),
                "gemv_hyper: y [M, N]");
    p.y = y->data_ptr();
    p.ldy = y->stride(0);
  }
  check_rc(nxd::gemv_hyper_launch((int)epi, p, cur_stream()), "gemv_hyper");
}

}  // namespace

PYBIND11_MODULE(_hybrid, m) {
  register_gemm(m);
  register_parallel(m);
  namespace py = pybind11;
  m.def("hyper_step", &hyper_step, py::arg("x"), py::arg("embed") = py::none(), py::arg("ids") = py::none(),
        py::arg("y") = py::none(), py::arg("bias") = py::none(), py::arg("mix") = py::none(), py::arg("write") = py::none(),
        py::arg("read") = py::none(), py::arg("norm_w") = py::none(), py::arg("eps") = 0.0, py::arg("h") = py::none(),
        py::arg("rows") = py::none(), py::arg("store") = true);
  m.def("relu_squared", &relu_squared);
  m.def("softcap_", &softcap_);
  m.def("delta_rule", &delta_rule, py::arg("proj"), py::arg("B"), py::arg("T"), py::arg("sizes"), py::arg("conv"),
        py::arg("a_log"), py::arg("dt_bias"), py::arg("norm_w"), py::arg("eps"), py::arg("pos"), py::arg("lens"),
        py::arg("slots"), py::arg("state"), py::arg("ring"), py::arg("y"), py::arg("fused") = true, py::arg("chunk_from") = 32);
  m.def("attn_prep", &attn_prep, py::arg("buf"), py::arg("B"), py::arg("T"), py::arg("sizes"), py::arg("bias"),
        py::arg("qn_w"), py::arg("kn_w"), py::arg("eps"), py::arg("cos"), py::arg("sin"), py::arg("pos"), py::arg("lens"),
        py::arg("slots"), py::arg("kc"), py::arg("vc"));
  m.def("window_attn", &window_attn, py::arg("buf"), py::arg("B"), py::arg("T"), py::arg("sizes"), py::arg("scale"),
        py::arg("softcap"), py::arg("window"), py::arg("lam"), py::arg("out_scale"), py::arg("out_eps"), py::arg("pos"),
        py::arg("lens"), py::arg("slots"), py::arg("kc"), py::arg("vc"), py::arg("y"), py::arg("from_buf"), py::arg("fused") = true);
  m.def("attn_decode", &attn_decode);
  m.def("pooled_prep", &pooled_prep);
  m.def("pooled_attn", &pooled_attn);
  m.def("pooled_decode", &pooled_decode);
  m.def("gemv_hyper", &gemv_hyper, py::arg("epi"), py::arg("x") = py::none(), py::arg("u") = py::none(),
        py::arg("norm_w") = py::none(), py::arg("eps") = 0.0, py::arg("w"), py::arg("y") = py::none(), py::arg("cap") = 0.0,
        py::arg("streams") = py::none(), py::arg("bias") = py::none(), py::arg("mix") = py::none(),
        py::arg("write") = py::none(), py::arg("read") = py::none(), py::arg("un") = py::none(), py::arg("alpha") = 1.0);
}
