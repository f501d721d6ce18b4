// Python bindings of mixers with a state per request, and of what surrounds
// them: short convolutions, selective scans, the gated delta rule, linear
// attention, row operations (substratus_amd._hybrid, see bindings.hip).
#include "bindings.h"

#include "add_norm.h"
#include "delta.h"
#include "gla.h"
#include "scan.h"
#include "short_conv.h"

#include <algorithm>

namespace {

// Number of entries, with state slots, positions and seq_start checked.
int check_entries(const Tensor& state_slots, const Tensor& positions,
                  const OptTensor& seq_start, long rows) {
  check(state_slots, torch::kInt32, "state_slots");
  check(positions, torch::kInt32, "positions");
  TORCH_CHECK(positions.numel() == rows, "one position per row");
  const int entries = state_slots.numel();
  if (seq_start) {
    check(*seq_start, torch::kInt32, "seq_start");
    TORCH_CHECK(seq_start->numel() == entries + 1, "entries differ");
  } else {
    TORCH_CHECK(rows == entries, "one row per entry");
  }
  return entries;
}

void check_f32(const Tensor& t, long n, const char* name) {
  check(t, torch::kFloat32, name);
  TORCH_CHECK(t.numel() == n, name, " must have ", n, " elements, has ",
              t.numel());
}

// [rows, n] view of activations
template <class T>
void check_view(const Tensor& t, long rows, long n, const char* name) {
  check_rows(t, Scalar<T>::type, name);
  TORCH_CHECK(t.size(0) == rows && t.size(1) == n, name, " must be [", rows,
              ", ", n, "]");
}

void add_norm(Tensor y, Tensor x, bool fresh, OptTensor rows, OptTensor pool,
              OptTensor at, OptTensor wt, OptTensor tokens, OptTensor table,
              double scale, OptTensor vec, Tensor w, OptTensor b, double eps) {
  const long n = x.size(0);
  const int width = x.size(1);
  check(x, torch::kFloat32, "x");
  check_f32(w, width, "w");
  if (b) check_f32(*b, width, "b");
  if (vec) check_f32(*vec, width, "vec");
  TORCH_CHECK(width <= add_norm_max_width(width), "row too wide");
  TORCH_CHECK(y.sizes() == x.sizes() && (!rows || rows->sizes() == x.sizes()),
              "add_norm: shapes differ");
  TORCH_CHECK(pool.has_value() == at.has_value() &&
              pool.has_value() == wt.has_value(),
              "picked rows need their places and weights");
  if (pool) {
    check(*at, torch::kInt32, "at");
    check(*wt, torch::kFloat32, "weights");
    TORCH_CHECK(at->dim() == 2 && at->size(0) == n && at->size(1) > 0 &&
                at->sizes() == wt->sizes() && pool->size(-1) == width,
                "picks differ");
  }
  TORCH_CHECK(tokens.has_value() == table.has_value(), "tokens need a table");
  if (table) {
    check(*tokens, torch::kInt32, "tokens");
    TORCH_CHECK(tokens->numel() == n && table->size(1) == width,
                "one token per row");
  }
  if (n == 0) return;
  by_type(y, [&](auto tag) {
    using T = decltype(tag);
    check(y, Scalar<T>::type, "y");
    for (const OptTensor* t : {&rows, &pool, &table})
      if (*t) check(**t, Scalar<T>::type, "addends");
    AddNorm<T> a{};
    a.y = ptr<T>(y); a.x = ptr<float>(x); a.fresh = fresh;
    a.rows = ptr<T>(rows); a.pool = ptr<T>(pool); a.at = ptr<int>(at);
    a.wt = ptr<float>(wt); a.picks = at ? at->size(1) : 0;
    a.tokens = ptr<int>(tokens); a.table = ptr<T>(table);
    a.vocab = table ? table->size(0) : 0; a.scale = scale;
    a.vec = ptr<float>(vec); a.w = ptr<float>(w); a.b = ptr<float>(b);
    a.width = width; a.eps = eps;
    launch_add_norm<T>(a, n, stream());
  });
  post("add_norm");
}

void joint_gate(Tensor out, Tensor o, Tensor norm, Tensor gate, double eps) {
  const long rows = o.size(0), n = o.size(1);
  check_f32(norm, n, "norm");
  if (rows == 0) return;
  by_type(o, [&](auto tag) {
    using T = decltype(tag);
    check(o, Scalar<T>::type, "o");
    check_view<T>(out, rows, n, "out");
    check_view<T>(gate, rows, n, "gate");
    launch_joint_gate<T>(ptr<T>(out), out.stride(0), ptr<T>(o),
                         ptr<float>(norm), ptr<T>(gate), gate.stride(0), rows,
                         n, eps, stream());
  });
  post("joint_gate");
}

void glu(Tensor out, Tensor x, const std::string& act, double limit) {
  const long rows = out.size(0), f = out.size(1);
  const Glu kind = glu_of(act);
  if (rows == 0 || f == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check_view<T>(out, rows, f, "out");
    check_view<T>(x, rows, 2 * f, "x");
    launch_glu<T>(ptr<T>(out), out.stride(0), ptr<T>(x), x.stride(0), rows, f,
                  kind, limit, stream());
  });
  post("glu");
}

void softcap(Tensor x, double cap) {
  if (x.numel() == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check(x, Scalar<T>::type, "x");
    launch_softcap<T>(ptr<T>(x), x.numel(), cap, stream());
  });
  post("softcap");
}

// out [rows, half, 2]
void rope_table(Tensor out, Tensor positions, Tensor turns) {
  const long rows = positions.numel(), half = turns.numel();
  check(positions, torch::kInt32, "positions");
  check(turns, torch::kFloat64, "turns");
  check_f32(out, rows * half * 2, "out");
  if (rows * half == 0) return;
  launch_rope_table(ptr<float>(out), ptr<int>(positions), ptr<double>(turns),
                    rows, half, stream());
  post("rope_table");
}

// What both convolutions take: x [rows, channels or more], weight [channels,
// taps], state [slots, taps - 1, channels].
template <class T>
Conv<T> conv(const Tensor& x, const OptTensor& in_bias, const Tensor& weight,
             const Tensor& state, const Tensor& state_slots,
             const Tensor& positions, const OptTensor& seq_start) {
  const long channels = weight.size(0), taps = weight.size(1);
  check_rows(x, Scalar<T>::type, "x");
  check(weight, torch::kFloat32, "weight");
  check(state, Scalar<T>::type, "state");
  if (in_bias) check_f32(*in_bias, channels, "in_bias");
  TORCH_CHECK(taps > 0 && x.size(1) >= channels && state.dim() == 3 &&
              state.size(1) == taps - 1 && state.size(2) == channels,
              "convolution: shapes differ");
  Conv<T> a{};
  a.x = ptr<T>(x); a.ld = x.stride(0); a.in_bias = ptr<float>(in_bias);
  a.weight = ptr<float>(weight); a.state = ptr<T>(state);
  a.state_slots = ptr<int>(state_slots); a.positions = ptr<int>(positions);
  a.seq_start = ptr<int>(seq_start);
  a.channels = channels; a.taps = taps;
  return a;
}

void short_conv(Tensor out, Tensor x, OptTensor in_bias, Tensor weight,
                OptTensor bias, bool act, Tensor state, Tensor state_slots,
                Tensor positions, OptTensor seq_start, int64_t max_len) {
  const long rows = x.size(0);
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  if (bias) check_f32(*bias, weight.size(0), "bias");
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    auto a = conv<T>(x, in_bias, weight, state, state_slots, positions,
                     seq_start);
    check(out, Scalar<T>::type, "out");
    TORCH_CHECK(out.size(0) == rows && out.size(1) == a.channels &&
                x.size(1) == a.channels, "out must be [rows, channels]");
    a.out = ptr<T>(out); a.bias = ptr<float>(bias); a.act = act;
    launch_short_conv<T>(a, entries, seq_start ? max_len : 1, stream());
  });
  post("short_conv");
}

void conv_rope(Tensor q, Tensor x, OptTensor in_bias, Tensor weight,
               Tensor state, Tensor state_slots, Tensor rope, Tensor kc,
               Tensor vc, Tensor positions, Tensor slots, OptTensor seq_start,
               int64_t max_len) {
  const long rows = x.size(0), kv = kc.size(1), dim = kc.size(3);
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  check(slots, torch::kInt32, "slots");
  check(rope, torch::kFloat32, "rope");
  TORCH_CHECK(slots.numel() == rows && rope.dim() == 3 &&
              rope.size(0) == rows && rope.size(2) == 2 &&
              2 * rope.size(1) <= dim, "conv_rope: rows differ");
  TORCH_CHECK(kc.sizes() == vc.sizes(), "caches differ");
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    auto a = conv<T>(x, in_bias, weight, state, state_slots, positions,
                     seq_start);
    check(q, Scalar<T>::type, "q");
    check(kc, Scalar<T>::type, "kc");
    check(vc, Scalar<T>::type, "vc");
    TORCH_CHECK(a.channels % dim == 0 && a.channels > kv * dim &&
                q.size(0) == rows && q.size(1) == a.channels - kv * dim,
                "q must be [rows, query heads * dim]");
    a.q = ptr<T>(q); a.kc = ptr<T>(kc); a.vc = ptr<T>(vc);
    a.rope = ptr<float>(rope); a.slots = ptr<int>(slots);
    a.half = rope.size(1); a.kv = kv; a.dim = dim; a.block_size = kc.size(2);
    launch_conv_rope<T>(a, entries, seq_start ? max_len : 1, stream());
  });
  post("conv_rope");
}

void conv_qkv(Tensor q, Tensor x, OptTensor in_bias, Tensor weight,
              Tensor state, Tensor state_slots, Tensor kc, Tensor vc,
              Tensor positions, Tensor slots, OptTensor seq_start, double temp,
              int64_t every, double v_eps, int64_t max_len) {
  const long rows = x.size(0), kv = kc.size(1), dim = kc.size(3),
             vdim = vc.size(3);
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(slots.numel() == rows, "one slot per row");
  TORCH_CHECK(kc.size(0) == vc.size(0) && kv == vc.size(1) &&
              kc.size(2) == vc.size(2), "caches differ");
  TORCH_CHECK(every > 0 && every < 1l << 31, "a temperature's steps");
  TORCH_CHECK(conv_qkv_takes(vdim), "values too wide");
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    auto a = conv<T>(x, in_bias, weight, state, state_slots, positions,
                     seq_start);
    check(q, Scalar<T>::type, "q");
    check(kc, Scalar<T>::type, "kc");
    check(vc, Scalar<T>::type, "vc");
    const long nq = a.channels - kv * (dim + vdim);
    TORCH_CHECK(nq > 0 && nq % dim == 0 && q.size(0) == rows &&
                q.size(1) == nq, "q must be [rows, query heads * dim]");
    a.q = ptr<T>(q); a.kc = ptr<T>(kc); a.vc = ptr<T>(vc);
    a.slots = ptr<int>(slots);
    a.kv = kv; a.dim = dim; a.vdim = vdim; a.block_size = kc.size(2);
    a.temp = temp; a.every = every; a.v_eps = v_eps;
    launch_conv_qkv<T>(a, entries, seq_start ? max_len : 1, stream());
  });
  post("conv_qkv");
}

void selective_scan(Tensor out, Tensor u, Tensor gate, Tensor z, Tensor zb,
                    Tensor low, int64_t b_at, Tensor a_, Tensor d,
                    Tensor state, Tensor state_slots, Tensor positions,
                    OptTensor seq_start, int64_t max_len, bool recurrent) {
  const long rows = u.size(0), channels = u.size(1), n = a_.size(1);
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  check_f32(z, rows * channels, "z");
  check_f32(zb, channels, "z_bias");
  check_f32(a_, channels * n, "a");
  check_f32(d, channels, "d");
  check(state, torch::kFloat32, "state");
  TORCH_CHECK(state.dim() == 3 && state.size(1) == channels &&
              state.size(2) == n, "state must be [slots, channels, n]");
  TORCH_CHECK(n > 0 && n <= SCAN_MAX_STATE, "state size over ",
              SCAN_MAX_STATE);
  TORCH_CHECK(low.size(0) == rows && b_at >= 0 && b_at + 2 * n <= low.size(1),
              "low is too narrow");
  if (rows == 0) return;
  by_type(u, [&](auto tag) {
    using T = decltype(tag);
    check(u, Scalar<T>::type, "u");
    check_view<T>(out, rows, channels, "out");
    check_view<T>(gate, rows, channels, "gate");
    check_rows(low, Scalar<T>::type, "low");
    Scan<T> a{};
    a.out = ptr<T>(out); a.u = ptr<T>(u); a.gate = ptr<T>(gate);
    a.z = ptr<float>(z); a.zb = ptr<float>(zb); a.low = ptr<T>(low) + b_at;
    a.a = ptr<float>(a_); a.d = ptr<float>(d); a.state = ptr<float>(state);
    a.state_slots = ptr<int>(state_slots); a.positions = ptr<int>(positions);
    a.seq_start = ptr<int>(seq_start);
    a.out_ld = out.stride(0); a.g_ld = gate.stride(0);
    a.low_ld = low.stride(0); a.channels = channels; a.n = n;
    const int longest = seq_start ? max_len : 1;
    const int nseg = recurrent ? 1
        : scan_segments(entries, channels, n, longest);
    Tensor ws, wd;
    if (nseg > 1) {
      ws = torch::empty({entries, nseg, channels, n}, state.options());
      wd = torch::empty({entries, nseg, channels}, state.options());
    }
    launch_scan<T>(a, entries, longest, nseg,
                   nseg > 1 ? ptr<float>(ws) : nullptr,
                   nseg > 1 ? ptr<float>(wd) : nullptr, stream());
  });
  post("selective_scan");
}

constexpr int DELTA_CHUNK_FROM = 8;             // tokens of a portion
constexpr long DELTA_WORKSPACE = 2l << 30;      // bytes

void delta(Tensor out, Tensor qkv, Tensor z, Tensor zb, Tensor rate,
           Tensor beta, Tensor norm, Tensor gate, Tensor state,
           Tensor state_slots, Tensor positions, OptTensor seq_start,
           int64_t kv_heads, double eps, double mult, int64_t max_len,
           bool recurrent) {
  const int heads = state.size(1), dim = state.size(2), vdim = state.size(3);
  const long rows = qkv.size(0);
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  check(state, torch::kFloat32, "state");
  check_f32(z, rows * heads * dim, "z");
  check_f32(zb, heads * dim, "z_bias");
  check_f32(rate, heads, "rate");
  check_f32(norm, vdim, "norm");
  TORCH_CHECK(kv_heads > 0 && heads % kv_heads == 0 &&
              qkv.size(1) == 2 * kv_heads * dim + heads * vdim,
              "delta: qkv must be [rows, q | k | v]");
  TORCH_CHECK(dim <= 1024 && vdim <= 2048, "head size over 1024, 2048");
  if (rows == 0) return;
  by_type(qkv, [&](auto tag) {
    using T = decltype(tag);
    check(qkv, Scalar<T>::type, "qkv");
    check_view<T>(out, rows, heads * vdim, "out");
    check_view<T>(gate, rows, heads * vdim, "gate");
    check_view<T>(beta, rows, heads, "beta");
    Delta<T> a{};
    a.out = ptr<T>(out); a.qkv = ptr<T>(qkv); a.z = ptr<float>(z);
    a.zb = ptr<float>(zb); a.rate = ptr<float>(rate); a.beta = ptr<T>(beta);
    a.gate = ptr<T>(gate); a.norm = ptr<float>(norm);
    a.state = ptr<float>(state); a.state_slots = ptr<int>(state_slots);
    a.positions = ptr<int>(positions); a.seq_start = ptr<int>(seq_start);
    a.ld = qkv.stride(0); a.out_ld = out.stride(0); a.b_ld = beta.stride(0);
    a.g_ld = gate.stride(0);
    a.heads = heads; a.kv_heads = kv_heads; a.dim = dim; a.vdim = vdim;
    a.eps = eps; a.mult = mult;
    if constexpr (std::is_same_v<T, bf16_t>) {
      if (seq_start && !recurrent && max_len >= DELTA_CHUNK_FROM &&
          delta_chunk_supported(a, max_len)) {
        TORCH_CHECK(entries <= 65535, "too many portions");
        const long bytes = delta_chunk_bytes(dim, rows, entries);
        const int some = std::clamp<long>(DELTA_WORKSPACE / bytes, 1, heads);
        Tensor ws = torch::empty({some * bytes},
                                 state.options().dtype(torch::kUInt8));
        for (int h0 = 0; h0 < heads; h0 += some)
          launch_delta_chunk(a, entries, max_len, h0,
                             std::min(some, heads - h0), ws.data_ptr(),
                             stream());
        return;
      }
    }
    launch_delta_recurrent<T>(a, entries, stream());
  });
  post("delta");
}

// Portions by chunks where the sizes allow, else token by token.
template <class T>
void run_gla(const Gla<T>& a, const Tensor& state, int entries,
             const OptTensor& seq_start, int64_t max_len, bool recurrent) {
  if constexpr (std::is_same_v<T, bf16_t>) {
    // the chunk kernel addresses a segment's rows with 32-bit offsets
    if (seq_start && !recurrent &&
        gla_chunk_supported(a.dim, a.vdim, a.rank) &&
        max_len * a.ld * 2 < 0x7ffffff0 - (1 << 20)) {
      const int nseg = gla_chunk_segments(entries, a.heads, max_len);
      Tensor ws, wd;
      if (nseg > 1) {
        ws = torch::empty({entries, nseg, a.heads, a.dim, a.vdim},
                          state.options());
        wd = torch::empty({entries, nseg, a.heads, a.dim}, state.options());
      }
      launch_gla_chunk(a, entries, max_len, nseg,
                       nseg > 1 ? ptr<float>(ws) : nullptr,
                       nseg > 1 ? ptr<float>(wd) : nullptr, stream());
      return;
    }
  }
  launch_gla_recurrent<T>(a, entries, stream());
}

// x [rows, >= q | k | v | g | A1 h]; state [slots, heads, dim, vdim]
void gla(Tensor out, Tensor x, Tensor a2, Tensor a2b, Tensor norm,
         Tensor state, Tensor state_slots, Tensor positions,
         OptTensor seq_start, double inv_tau, double eps, int64_t max_len,
         bool recurrent) {
  const int heads = state.size(1), dim = state.size(2), vdim = state.size(3);
  const int rank = a2.size(1);
  const long rows = x.size(0);
  check(a2, torch::kFloat32, "a2");
  check(a2b, torch::kFloat32, "a2b");
  check(norm, torch::kFloat32, "norm");
  check(state, torch::kFloat32, "state");
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  TORCH_CHECK(a2.size(0) == heads * dim && a2b.numel() == heads * dim &&
              norm.numel() == vdim && positions.numel() == rows,
              "gla: shapes differ");
  TORCH_CHECK(x.size(1) >= 2 * heads * (dim + vdim) + rank, "x too narrow");
  TORCH_CHECK(dim <= 2048 && vdim <= 2048, "head size over 2048");
  TORCH_CHECK(out.size(0) == rows && out.size(1) == heads * vdim,
              "out must be [rows, heads * vdim]");
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check_rows(x, Scalar<T>::type, "x");
    check(out, Scalar<T>::type, "out");
    Gla<T> a{};
    a.out = ptr<T>(out); a.x = ptr<T>(x); a.ld = x.stride(0);
    a.k_off = heads * dim; a.v_off = 2 * heads * dim;
    a.g_off = a.v_off + heads * vdim; a.a_off = a.g_off + heads * vdim;
    a.a2 = ptr<float>(a2); a.a2b = ptr<float>(a2b);
    a.norm = ptr<float>(norm); a.state = ptr<float>(state);
    a.state_slots = ptr<int>(state_slots);
    a.positions = ptr<int>(positions); a.seq_start = ptr<int>(seq_start);
    a.heads = heads; a.dim = dim; a.vdim = vdim; a.rank = rank;
    a.qscale = 1.f / std::sqrt((float)dim); a.inv_tau = inv_tau; a.eps = eps;
    run_gla<T>(a, state, entries, seq_start, max_len, recurrent);
  });
  post("gla");
}

// x [rows, >= q | k | v], which pass silu; constant decays [heads]
void lightning(Tensor out, Tensor x, Tensor decay, Tensor state,
               Tensor state_slots, Tensor positions, OptTensor seq_start,
               int64_t max_len, bool recurrent) {
  const int heads = state.size(1), dim = state.size(2), vdim = state.size(3);
  const long rows = x.size(0);
  const int entries = check_entries(state_slots, positions, seq_start, rows);
  check_f32(decay, heads, "decay");
  check(state, torch::kFloat32, "state");
  TORCH_CHECK(x.size(1) >= heads * (2 * dim + vdim), "x too narrow");
  TORCH_CHECK(dim <= 2048 && vdim <= 2048, "head size over 2048");
  TORCH_CHECK(out.size(0) == rows && out.size(1) == heads * vdim,
              "out must be [rows, heads * vdim]");
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check_rows(x, Scalar<T>::type, "x");
    check(out, Scalar<T>::type, "out");
    Gla<T> a{};
    a.out = ptr<T>(out); a.x = ptr<T>(x); a.ld = x.stride(0);
    a.k_off = heads * dim; a.v_off = 2 * heads * dim;
    a.decay = ptr<float>(decay); a.state = ptr<float>(state);
    a.state_slots = ptr<int>(state_slots);
    a.positions = ptr<int>(positions); a.seq_start = ptr<int>(seq_start);
    a.heads = heads; a.dim = dim; a.vdim = vdim;
    a.qscale = 1.f;
    run_gla<T>(a, state, entries, seq_start, max_len, recurrent);
  });
  post("lightning");
}

}  // namespace

void bind_mixers(pybind11::module& m) {
  m.def("add_norm", &add_norm);
  m.def("joint_gate", &joint_gate);
  m.def("glu", &glu);
  m.def("softcap", &softcap);
  m.def("rope_table", &rope_table);
  m.def("short_conv", &short_conv);
  m.def("conv_rope", &conv_rope);
  m.def("conv_qkv", &conv_qkv);
  m.def("selective_scan", &selective_scan);
  m.def("delta", &delta);
  m.def("gla", &gla);
  m.def("lightning", &lightning);
}
