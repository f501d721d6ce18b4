// Python bindings of the hybrid-model kernels (substratus_amd._hybrid): norms
// of a 32-bit residual, cache-reading attention, mixtures of experts; mixers
// with a state per request are in bindings_mixers.hip.
// Every op takes float or bf16 activations. Shapes are checked here; kernels
// are thin and trusting.
#include "bindings.h"

#include <numeric>

#include "attention_ctx.h"
#include "group_gemm.h"

template <class T>
void launch_stream_norm(T*, float*, const T*, const int*, const float*, int, const float*, const float*, long, int, float, float, float, float, hipStream_t);
template <class T>
void launch_latent_prepare(T*, long, int, int, int, int, int, const float*, float, const double*, int, const int*, T*, const int*, const float*, int, long, hipStream_t);
void launch_latent_gather(void*, void*, const void*, int, int, int, const int*, int, const int*, const int*, const int*, int, int, int, int, hipStream_t);
int moe_max_experts();
void launch_moe_select(int*, float*, const float*, int, int, int, int, int, int, const float*, bool, bool, const float*, int, hipStream_t);
void launch_moe_sort(int*, int*, int*, int*, const int*, int, int, int, int, hipStream_t);
template <class T>
void launch_embed_norm(T*, float*, const T*, const int*, float, const T*, const int*, int, const float*, long, int, int, float, float, hipStream_t);
int stream_norm_max_width(int width);
template <class T>
void launch_qkv_prepare(T*, long, int, int, int, const float*, const float*, float, const T*, long, const float*, T*, T*, const int*, long, int, int, hipStream_t);
void launch_silu_mul(bf16_t*, const bf16_t*, long, int, hipStream_t);
void launch_silu_mul_any(float*, const float*, long, int, hipStream_t);
void launch_silu_mul_any(bf16_t*, const bf16_t*, long, int, hipStream_t);

namespace {

// rows [pool, width], picked by at and weights [rows of x, picks], or
// [rows of x, width] without those
void stream_norm(Tensor y, Tensor x, Tensor rows, OptTensor at,
                 OptTensor weights, Tensor w_post, OptTensor w_pre, double off,
                 double eps, double out_scale, double mult) {
  const int width = x.size(-1);
  const long n = x.numel() / width;
  check(x, torch::kFloat32, "x");
  check(w_post, torch::kFloat32, "w_post");
  TORCH_CHECK(width <= stream_norm_max_width(width), "row too wide");
  TORCH_CHECK(y.numel() == x.numel() && w_post.numel() == width &&
              rows.size(-1) == width, "stream_norm: shapes differ");
  if (w_pre) {
    check(*w_pre, torch::kFloat32, "w_pre");
    TORCH_CHECK(w_pre->numel() == width, "stream_norm: shapes differ");
  }
  TORCH_CHECK(at.has_value() == weights.has_value(), "at needs weights");
  int picks = 0;
  if (at) {
    check(*at, torch::kInt32, "at");
    check(*weights, torch::kFloat32, "weights");
    TORCH_CHECK(at->dim() == 2 && at->size(0) == n &&
                at->sizes() == weights->sizes(), "picks differ");
    picks = at->size(1);
  } else {
    TORCH_CHECK(rows.numel() == x.numel(), "stream_norm: shapes differ");
  }
  if (n == 0) return;
  by_type(y, [&](auto tag) {
    using T = decltype(tag);
    check(y, Scalar<T>::type, "y");
    check(rows, Scalar<T>::type, "delta");
    launch_stream_norm<T>(ptr<T>(y), ptr<float>(x), ptr<T>(rows), ptr<int>(at),
                          ptr<float>(weights), picks, ptr<float>(w_post),
                          ptr<float>(w_pre), n, width, off, eps, out_scale,
                          mult, stream());
  });
  post("stream_norm");
}

void embed_norm(Tensor y, Tensor x, Tensor table, Tensor tokens,
                OptTensor w_pre, double off, double eps, double scale,
                OptTensor pos, OptTensor positions) {
  const int width = table.size(1);
  const long rows = tokens.numel();
  check(x, torch::kFloat32, "x");
  check(tokens, torch::kInt32, "tokens");
  TORCH_CHECK(width <= stream_norm_max_width(width), "row too wide");
  TORCH_CHECK(y.numel() == rows * width && x.numel() == rows * width,
              "embed_norm: shapes differ");
  if (w_pre) {
    check(*w_pre, torch::kFloat32, "w_pre");
    TORCH_CHECK(w_pre->numel() == width, "embed_norm: shapes differ");
  }
  TORCH_CHECK(pos.has_value() == positions.has_value(),
              "positions need their vectors");
  if (pos) {
    check(*positions, torch::kInt32, "positions");
    TORCH_CHECK(positions->numel() == rows && pos->dim() == 2 &&
                pos->size(0) > 0 && pos->size(1) == width,
                "embed_norm: shapes differ");
  }
  if (rows == 0) return;
  by_type(y, [&](auto tag) {
    using T = decltype(tag);
    check(y, Scalar<T>::type, "y");
    check(table, Scalar<T>::type, "table");
    if (pos) check(*pos, Scalar<T>::type, "pos");
    launch_embed_norm<T>(ptr<T>(y), ptr<float>(x), ptr<T>(table),
                         ptr<int>(tokens), scale, ptr<T>(pos),
                         ptr<int>(positions), pos ? pos->size(0) : 0,
                         ptr<float>(w_pre), rows, width, table.size(0), off,
                         eps, stream());
  });
  post("embed_norm");
}

// buf [rows, >= nq + nk + nv]; kc [blocks, kv_heads, block, dim]
void qkv_prepare(Tensor buf, int64_t nq, OptTensor qw, OptTensor kw,
                 double eps, OptTensor v_first, OptTensor lam, Tensor kc,
                 Tensor vc, Tensor slots) {
  const int kv = kc.size(1), nk = kv * kc.size(3), nv = kv * vc.size(3);
  const long rows = buf.size(0);
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(slots.numel() == rows, "one slot per row");
  TORCH_CHECK(buf.size(1) >= nq + nk + nv, "buf too narrow");
  TORCH_CHECK(kc.size(0) == vc.size(0) && kc.size(1) == vc.size(1) &&
              kc.size(2) == vc.size(2), "caches differ");
  TORCH_CHECK(qw.has_value() == kw.has_value(), "norm both or neither");
  if (qw) {
    check(*qw, torch::kFloat32, "qw");
    check(*kw, torch::kFloat32, "kw");
    TORCH_CHECK(qw->numel() == nq && kw->numel() == nk, "norm weight sizes");
  }
  if (v_first) {
    TORCH_CHECK(lam.has_value() && lam->numel() == 1, "v_first needs lam");
    check(*lam, torch::kFloat32, "lam");
    TORCH_CHECK(v_first->size(0) == rows && v_first->size(1) == nv,
                "v_first must be [rows, nv]");
  }
  if (rows == 0) return;
  by_type(buf, [&](auto tag) {
    using T = decltype(tag);
    check_rows(buf, Scalar<T>::type, "buf");
    check(kc, Scalar<T>::type, "kc");
    check(vc, Scalar<T>::type, "vc");
    if (v_first) check_rows(*v_first, Scalar<T>::type, "v_first");
    launch_qkv_prepare<T>(ptr<T>(buf), buf.stride(0), nq, nk, nv,
                          ptr<float>(qw), ptr<float>(kw), eps,
                          ptr<T>(v_first), v_first ? v_first->stride(0) : 0,
                          ptr<float>(lam), ptr<T>(kc), ptr<T>(vc),
                          ptr<int>(slots), rows, kv, kc.size(2), stream());
  });
  post("qkv_prepare");
}

// One entry per row (seq_start absent) or portions of up to max_len rows.
// `rows` are those of q; span: most keys a row can see; any: take the
// untiled kernel.
void attn_ctx(Tensor out, Tensor q, OptTensor gate, Tensor kc, Tensor vc,
              OptTensor bias, OptTensor sink, Tensor positions,
              OptTensor seq_start, Tensor block_table, double scale,
              int64_t chunk, int64_t window, int64_t keep, double cap,
              double mult, int64_t max_len, int64_t span, bool any,
              OptTensor r1, OptTensor r2, OptTensor wbias) {
  const int kv = kc.size(1), dim = kc.size(3), vdim = vc.size(3);
  const long rows = q.size(0);
  TORCH_CHECK(q.size(1) % dim == 0, "q is not heads * dim wide");
  const int heads = q.size(1) / dim;
  TORCH_CHECK(heads % kv == 0, "query heads must divide by kv heads");
  TORCH_CHECK(vdim <= ATTN_ANY_VDIM, "value size over ", ATTN_ANY_VDIM);
  TORCH_CHECK(dim <= 8192, "key size over 8192");
  TORCH_CHECK(vc.size(0) == kc.size(0) && vc.size(1) == kv &&
              vc.size(2) == kc.size(2), "caches differ");
  TORCH_CHECK(out.size(0) == rows && out.size(1) == heads * vdim,
              "out must be [rows, heads * vdim]");
  check(positions, torch::kInt32, "positions");
  check(block_table, torch::kInt32, "block_table");
  TORCH_CHECK(positions.numel() == rows, "one position per row");
  const int entries = block_table.size(0);
  if (seq_start) {
    check(*seq_start, torch::kInt32, "seq_start");
    TORCH_CHECK(seq_start->numel() == entries + 1, "entries differ");
  } else {
    TORCH_CHECK(rows == entries, "one row per entry");
  }
  if (bias) {
    check(*bias, torch::kFloat32, "bias");
    TORCH_CHECK(bias->dim() == 2 && bias->size(0) == heads, "bias heads");
  }
  if (sink) {
    check(*sink, torch::kFloat32, "sink");
    TORCH_CHECK(sink->numel() == heads, "sink heads");
  }
  TORCH_CHECK(r1.has_value() == r2.has_value(), "r1 needs r2");
  for (const OptTensor* t : {&r1, &r2, &wbias})
    if (*t) {
      check(**t, torch::kFloat32, "numbers per head");
      TORCH_CHECK((*t)->numel() == heads, "one number per head");
    }
  TORCH_CHECK(!wbias || !sink, "sigmoid weights have no sink");
  TORCH_CHECK(chunk == 0 || window == 0, "a chunk or a window, not both");
  if (rows == 0) return;
  by_type(q, [&](auto tag) {
    using T = decltype(tag);
    check_rows(q, Scalar<T>::type, "q");
    check_rows(out, Scalar<T>::type, "out");
    check(kc, Scalar<T>::type, "kc");
    // values may be the first columns of wider rows
    check(vc, Scalar<T>::type, "vc", false);
    const long v_ld = vc.stride(2);
    TORCH_CHECK(vc.stride(3) == 1 && v_ld >= vdim &&
                vc.stride(1) == v_ld * vc.size(2) &&
                vc.stride(0) == vc.stride(1) * kv,
                "vc rows must be equally far apart");
    if (gate) {
      check_rows(*gate, Scalar<T>::type, "gate");
      TORCH_CHECK(gate->size(0) == rows && gate->size(1) == heads,
                  "gate must be [rows, heads]");
    }
    AttnCtx<T> a{};
    a.out = ptr<T>(out); a.q = ptr<T>(q); a.gate = ptr<T>(gate);
    a.kc = ptr<T>(kc); a.vc = ptr<T>(vc); a.bias = ptr<float>(bias);
    a.positions = ptr<int>(positions); a.seq_start = ptr<int>(seq_start);
    a.block_table = ptr<int>(block_table);
    a.v_ld = v_ld;
    a.q_ld = q.stride(0); a.g_ld = gate ? gate->stride(0) : 0;
    a.heads = heads; a.kv_heads = kv; a.dim = dim; a.vdim = vdim;
    a.nbias = bias ? bias->size(1) : 1; a.chunk = chunk;
    a.max_blocks = block_table.size(1); a.block_size = kc.size(2);
    a.scale = scale;
    a.sink = ptr<float>(sink);
    a.r1 = ptr<float>(r1); a.r2 = ptr<float>(r2);
    a.wbias = ptr<float>(wbias);
    a.window = window; a.keep = window > 0 ? keep : 0;
    a.cap = cap; a.mult = mult;
    a.out_ld = out.stride(0);
    a.quads = vdim % 4 == 0 && a.out_ld % 4 == 0 &&
              reinterpret_cast<uintptr_t>(a.out) % (4 * sizeof(T)) == 0;
    if constexpr (std::is_same_v<T, bf16_t>) {
      // the tiled kernels read q rows in 16-byte pieces
      const bool aligned = a.q_ld % 8 == 0 &&
          reinterpret_cast<uintptr_t>(a.q) % 16 == 0;
      any = any || v_ld % 8 != 0;
      if (!any && aligned && kv == 1 && a.kc == a.vc && v_ld == dim && !bias &&
          !gate && chunk == 0 && a.keep == 0 && !sink && !r1 && !wbias &&
          cap == 0 && mult == 1 && out.is_contiguous() &&
          attn_latent_supported(dim, vdim, a.block_size)) {
        const int longest = seq_start ? max_len : 1;
        const int splits = attn_latent_splits(entries, longest, heads, span);
        Tensor po, pml;
        if (splits > 1) {
          const auto opt = out.options().dtype(torch::kFloat32);
          po = torch::empty({rows, heads, splits, vdim}, opt);
          pml = torch::empty({rows, heads, splits, 2}, opt);
        }
        launch_attn_latent(a, entries, longest, span, splits,
                           splits > 1 ? ptr<float>(po) : nullptr,
                           splits > 1 ? ptr<float>(pml) : nullptr, stream());
        if (splits > 1)
          launch_attn_ctx_merge(a, rows, splits, ptr<float>(po),
                                ptr<float>(pml), stream());
        return;
      }
      if (!any && seq_start && aligned && !(wbias && cap > 0) &&
          attn_ctx_prefill_supported(dim, vdim, a.block_size)) {
        launch_attn_ctx_prefill(a, entries, max_len, stream());
        return;
      }
      if (!any && !seq_start &&
          attn_ctx_decode_supported(dim, vdim, a.block_size)) {
        const int splits =
            attn_ctx_decode_splits(entries, heads, kv, span);
        Tensor po, pml;
        if (splits > 1) {
          const auto opt = out.options().dtype(torch::kFloat32);
          po = torch::empty({rows, heads, splits, vdim}, opt);
          pml = torch::empty({rows, heads, splits, 2}, opt);
        }
        launch_attn_ctx_decode(a, entries, splits,
                               splits > 1 ? ptr<float>(po) : nullptr,
                               splits > 1 ? ptr<float>(pml) : nullptr,
                               stream());
        return;
      }
    }
    launch_attn_ctx_any<T>(a, entries, seq_start ? max_len : 1, stream());
  });
  post("attn_ctx");
}

// Portions over keys and values that lie unpaged, ctx_start[e + 1] -
// ctx_start[e] of them per entry: kv rows [keys of all heads | values of all
// heads], kr rows the key part that follows every head's own. With a window,
// an entry's first key is the first that its rows see. gate by column or by
// head.
void attn_flat(Tensor out, Tensor q, OptTensor gate, Tensor kv, Tensor kr,
               Tensor positions, Tensor seq_start, Tensor ctx_start,
               int64_t heads, int64_t vdim, double scale, int64_t window,
               int64_t max_len) {
  using T = bf16_t;
  const long rows = q.size(0), entries = seq_start.numel() - 1;
  const long dim = q.size(1) / heads, shared = kr.size(1);
  check_rows(q, Scalar<T>::type, "q");
  check(out, Scalar<T>::type, "out");
  check(kv, Scalar<T>::type, "kv");
  check(kr, Scalar<T>::type, "kr");
  check(positions, torch::kInt32, "positions");
  check(seq_start, torch::kInt32, "seq_start");
  check(ctx_start, torch::kInt32, "ctx_start");
  TORCH_CHECK(q.size(1) == heads * dim && kv.size(0) == kr.size(0) &&
              kv.size(1) == heads * (dim - shared + vdim) && shared < dim,
              "kv must be [keys, heads * (own + vdim)]");
  TORCH_CHECK(out.size(0) == rows && out.size(1) == heads * vdim &&
              positions.numel() == rows && ctx_start.numel() == entries + 1,
              "attn_flat: shapes differ");
  AttnCtx<T> a{};
  a.dim = dim; a.vdim = vdim; a.shared = shared;
  TORCH_CHECK(attn_ctx_prefill_supported(dim, vdim, 16) && shared % 8 == 0 &&
              q.stride(0) % 8 == 0 &&
              reinterpret_cast<uintptr_t>(q.data_ptr()) % 16 == 0,
              "attn_flat: sizes must be multiples of 8");
  if (gate) {
    check_rows(*gate, Scalar<T>::type, "gate");
    a.gate_each = gate->size(1) == heads * vdim;
    TORCH_CHECK(gate->size(0) == rows &&
                (gate->size(1) == heads ||
                 (a.gate_each && gate->stride(0) % 4 == 0 &&
                  reinterpret_cast<uintptr_t>(gate->data_ptr()) % 8 == 0)),
                "gate must be [rows, heads * vdim] or [rows, heads]");
  }
  if (rows == 0) return;
  a.out = ptr<T>(out); a.q = ptr<T>(q); a.gate = ptr<T>(gate);
  a.kc = ptr<T>(kv); a.vc = a.kc + heads * (dim - shared); a.kr = ptr<T>(kr);
  a.positions = ptr<int>(positions); a.seq_start = ptr<int>(seq_start);
  a.ctx_start = ptr<int>(ctx_start);
  a.q_ld = q.stride(0); a.g_ld = gate ? gate->stride(0) : 0;
  a.v_ld = kv.size(1);
  a.heads = a.kv_heads = heads; a.nbias = 1; a.block_size = 16;
  a.scale = scale; a.mult = 1.f; a.window = window;
  a.out_ld = out.stride(0); a.quads = vdim % 4 == 0;
  launch_attn_ctx_prefill(a, entries, max_len, stream());
  post("attn_flat");
}

// c [keys, rank] and kr [keys, rot] of what portions see, entry by entry
void latent_gather(Tensor c, Tensor kr, Tensor cache, Tensor block_table,
                   Tensor ctx_start, Tensor positions, Tensor seq_start,
                   int64_t window, int64_t max_len) {
  check(block_table, torch::kInt32, "block_table");
  check(positions, torch::kInt32, "positions");
  check(seq_start, torch::kInt32, "seq_start");
  check(ctx_start, torch::kInt32, "ctx_start");
  check(c, cache.scalar_type(), "c");
  check(kr, cache.scalar_type(), "kr");
  check(cache, cache.scalar_type(), "cache");
  const int entries = block_table.size(0);
  TORCH_CHECK(cache.size(1) == 1 && cache.size(3) == c.size(1) + kr.size(1) &&
              c.size(0) == kr.size(0) && ctx_start.numel() == entries + 1 &&
              seq_start.numel() == entries + 1,
              "latent_gather: shapes differ");
  if (entries == 0) return;
  launch_latent_gather(c.data_ptr(), kr.data_ptr(), cache.data_ptr(),
                       cache.element_size(), c.size(1), kr.size(1),
                       ptr<int>(block_table), block_table.size(1),
                       ptr<int>(ctx_start), ptr<int>(positions),
                       ptr<int>(seq_start), window, max_len, entries,
                       cache.size(2), stream());
  post("latent_gather");
}

// buf rows [queries | ... | latent | key part], the latter from column c_at
// on, or nowhere (-1); cache [blocks, 1, block, rank + rot_dim]. With q_norm,
// rows begin with the latent that queries are made of.
void latent_prepare(Tensor buf, int64_t heads, int64_t dim, int64_t rot_dim,
                    int64_t c_at, OptTensor norm, double eps, Tensor turns,
                    Tensor positions, Tensor cache, Tensor slots,
                    OptTensor q_norm) {
  const long rows = buf.size(0);
  const int half = turns.numel(), row = cache.size(3);
  const int rank = row - rot_dim;
  check(turns, torch::kFloat64, "turns");
  check(positions, torch::kInt32, "positions");
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(positions.numel() == rows && slots.numel() == rows,
              "one position and slot per row");
  TORCH_CHECK(2 * half <= rot_dim && half <= 4096, "too many turns");
  TORCH_CHECK(heads * (dim + rot_dim) <= buf.size(1), "buf too narrow");
  if (q_norm) {
    check(*q_norm, torch::kFloat32, "q_norm");
    TORCH_CHECK(heads == 0 && q_norm->numel() <= buf.size(1),
                "queries' latent: rows too narrow, or heads beside it");
  }
  TORCH_CHECK(rank > 0 && cache.size(1) == 1, "cache must hold latents");
  TORCH_CHECK((c_at >= 0) == norm.has_value(), "latents need their norm");
  if (norm) {
    check(*norm, torch::kFloat32, "norm");
    TORCH_CHECK(norm->numel() == rank, "norm size");
    TORCH_CHECK(c_at + row <= buf.size(1), "buf too narrow");
  }
  if (rows == 0) return;
  by_type(buf, [&](auto tag) {
    using T = decltype(tag);
    check_rows(buf, Scalar<T>::type, "buf");
    check(cache, Scalar<T>::type, "cache");
    launch_latent_prepare<T>(ptr<T>(buf), buf.stride(0), heads, dim, rot_dim,
                             c_at, rank, ptr<float>(norm), eps,
                             ptr<double>(turns), half, ptr<int>(positions),
                             ptr<T>(cache), ptr<int>(slots),
                             ptr<float>(q_norm), q_norm ? q_norm->numel() : 0,
                             rows, stream());
  });
  post("latent_prepare");
}

template <class T, class Y>
void group_gemm(const GroupGemm<T, Y>& a, int tile, const char* op) {
  TORCH_CHECK(a.tiles == nullptr || group_gemm_takes(a, tile), op,
              ": tiles of ", tile, " rows");
  launch_group_gemm<T, Y>(a, tile, stream());
  post(op);
}

template <class T, class Y = T>
GroupGemm<T, Y> product(const Tensor& y, const Tensor& x, const Tensor& w) {
  GroupGemm<T, Y> a{};
  check_rows(x, Scalar<T>::type, "x");
  check(y, Scalar<Y>::type, "y");
  check(w, Scalar<T>::type, "w");
  a.y = ptr<Y>(y); a.x = ptr<T>(x); a.w = ptr<T>(w);
  a.y_ld = y.stride(0); a.x_ld = x.stride(0);
  a.n = w.size(-2); a.k = w.size(-1);
  a.groups = w.dim() == 3 ? w.size(0) : 1;
  a.m = x.size(0);
  a.splits = 1;
  a.act = Act::NONE;
  return a;
}

// out [rows, heads, n + tail], x [rows, heads, k + tail] view, w [heads, n, k]
void head_linear(Tensor out, Tensor x, Tensor w, OptTensor gate,
                 int64_t tail) {
  const long rows = x.size(0), heads = w.size(0), n = w.size(1),
             k = w.size(2);
  TORCH_CHECK(x.dim() == 3 && x.size(1) == heads && x.size(2) == k + tail &&
              (x.stride(2) == 1 || x.size(2) == 1) && tail >= 0,
              "x must be [rows, heads, k + tail]");
  TORCH_CHECK(out.dim() == 3 && out.size(0) == rows && out.size(1) == heads &&
              out.size(2) == n + tail, "out must be [rows, heads, n + tail]");
  if (gate)
    TORCH_CHECK(gate->size(0) == rows && (gate->size(1) == heads * n ||
                                          gate->size(1) == heads),
                "gate must be [rows, heads * n] or [rows, heads]");
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check(x, Scalar<T>::type, "x", false);
    check(w, Scalar<T>::type, "w");
    check(out, Scalar<T>::type, "out");
    GroupGemm<T, T> a{};
    a.y = ptr<T>(out); a.x = ptr<T>(x); a.w = ptr<T>(w);
    a.y_ld = heads * (n + tail); a.y_gs = n + tail;
    a.x_ld = x.stride(0); a.x_gs = x.stride(1);
    a.m = rows; a.n = n; a.k = k; a.groups = heads; a.splits = 1;
    a.tail = tail;
    a.act = Act::NONE;
    if (gate) {
      check_rows(*gate, Scalar<T>::type, "gate");
      a.act = Act::GATE;
      a.gate = ptr<T>(gate); a.gate_ld = gate->stride(0);
      a.gate_each = gate->size(1) == heads * n;
      a.gate_gs = a.gate_each ? n : 1;
    }
    group_gemm(a, group_gemm_tile(rows, 1, std::is_same_v<T, bf16_t>, k),
               "head_linear");
  });
}

// Scores in float32, [splits, rows, experts]; sums over the first axis are
// left to moe_select.
Tensor router_scores(Tensor x, Tensor w) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == w.size(1),
              "router_scores: shapes differ");
  const auto opt = x.options().dtype(torch::kFloat32);
  const long rows = x.size(0), experts = w.size(0);
  if (rows == 0) return torch::empty({1, rows, experts}, opt);
  Tensor z;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    // its place in memory is not part of the choice of splits
    auto a = product<T, float>(torch::empty({0, experts}, opt), x, w);
    a.splits = group_gemm_splits(a);
    z = torch::empty({a.splits, rows, experts}, opt);
    a.y = ptr<float>(z);
    group_gemm(a, std::min(64, group_gemm_tile(
                   rows, 1, std::is_same_v<T, bf16_t>, w.size(1))),
               "router_scores");
  });
  return z;
}

// gelu_tanh(x w^T) * table[tokens, t_at : t_at + n]
void side_gate(Tensor out, Tensor x, Tensor w, Tensor tokens, Tensor table,
               int64_t t_at) {
  check(tokens, torch::kInt32, "tokens");
  TORCH_CHECK(x.size(1) == w.size(1) && out.size(0) == x.size(0) &&
              out.size(1) == w.size(0) && tokens.numel() == x.size(0),
              "side_gate: shapes differ");
  TORCH_CHECK(t_at >= 0 && t_at + w.size(0) <= table.size(1),
              "table too narrow");
  if (x.size(0) == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check(table, Scalar<T>::type, "table");
    auto a = product<T>(out, x, w);
    a.act = Act::SIDE;
    a.tokens = ptr<int>(tokens); a.table = ptr<T>(table) + t_at;
    a.t_ld = table.stride(0); a.vocab = table.size(0);
    group_gemm(a, std::min(128, group_gemm_tile(
                   x.size(0), 1, std::is_same_v<T, bf16_t>, w.size(1))),
               "side_gate");
  });
}

// x w^T in float32, unrounded
Tensor linear32(Tensor x, Tensor w) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && x.size(1) == w.size(1),
              "linear32: shapes differ");
  Tensor y = torch::empty({x.size(0), w.size(0)},
                          x.options().dtype(torch::kFloat32));
  if (x.size(0) == 0) return y;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    auto a = product<T, float>(y, x, w);
    group_gemm(a, std::min(128, group_gemm_tile(
                   x.size(0), 1, std::is_same_v<T, bf16_t>, w.size(1))),
               "linear32");
  });
  return y;
}

void moe_select(Tensor ids, Tensor weights, Tensor z, int64_t groups,
                int64_t keep, OptTensor bias, bool over_chosen, bool sigmoid,
                OptTensor correction, int64_t group_best) {
  TORCH_CHECK(z.dim() == 3, "z must be [splits, rows, experts]");
  const long rows = z.size(1), experts = z.size(2), top = ids.size(1);
  check(ids, torch::kInt32, "ids");
  check(weights, torch::kFloat32, "weights");
  check(z, torch::kFloat32, "z");
  TORCH_CHECK(ids.size(0) == rows && ids.sizes() == weights.sizes(),
              "moe_select: shapes differ");
  TORCH_CHECK(experts <= moe_max_experts(), "too many experts");
  if (bias) {
    check(*bias, torch::kFloat32, "bias");
    TORCH_CHECK(bias->numel() == experts, "one bias per expert");
  }
  if (correction) {
    check(*correction, torch::kFloat32, "correction");
    TORCH_CHECK(correction->numel() == experts, "one correction per expert");
  }
  TORCH_CHECK(group_best == 1 || group_best == 2,
              "a group's score is its best one or two");
  TORCH_CHECK(!(sigmoid && over_chosen), "sigmoid scores have no sum");
  TORCH_CHECK(groups > 0 && experts % groups == 0 && keep > 0 &&
              keep <= groups && top > 0 && top <= experts / groups * keep,
              "moe_select: cannot choose so many");
  if (rows == 0) return;
  launch_moe_select(ptr<int>(ids), ptr<float>(weights), ptr<float>(z),
                    z.size(0), rows, experts, top, groups, keep,
                    ptr<float>(bias), over_chosen, sigmoid,
                    ptr<float>(correction), group_best, stream());
  post("moe_select");
}

int64_t moe_tile(int64_t packed, int64_t experts, bool bf16, int64_t k,
                 int64_t n) {
  return group_gemm_tile(packed, experts, bf16, std::gcd(k, n));
}

// tiles: [1 + 2 * bound], of which each expert's last may be short
void moe_sort(Tensor at, Tensor src, Tensor start, Tensor tiles, Tensor ids,
              int64_t tile) {
  const long n = ids.numel(), experts = start.numel() - 1;
  for (const Tensor* t : {&at, &src, &start, &tiles, &ids})
    check(*t, torch::kInt32, "moe_sort tensors");
  TORCH_CHECK(at.numel() == n && src.numel() == n && tile > 0 &&
              experts > 0 && experts <= moe_max_experts(),
              "moe_sort: shapes differ");
  TORCH_CHECK(tiles.numel() >= 1 + 2 * ((n + tile - 1) / tile +
                                        std::min(experts, n)),
              "moe_sort: room for too few tiles");
  if (n == 0) return;
  launch_moe_sort(ptr<int>(at), ptr<int>(src), ptr<int>(start),
                  ptr<int>(tiles), ptr<int>(ids), n, ids.size(-1), experts,
                  tile, stream());
  post("moe_sort");
}

// Every packed row by its expert's matrix: out [packed, n], w [experts, n, k];
// packed row r is row src[r] of x, or row r. act: none, gelu, or a gated
// feed-forward's (w has the rows of gate and up in turn, out half as many
// columns).
void expert_linear(Tensor out, Tensor x, Tensor w, OptTensor src,
                   Tensor start, Tensor tiles, int64_t tile,
                   const std::string& act, double limit) {
  const bool glu = act != "none" && act != "gelu";
  check(start, torch::kInt32, "start");
  check(tiles, torch::kInt32, "tiles");
  TORCH_CHECK(w.dim() == 3 && start.numel() == w.size(0) + 1 &&
              x.size(1) == w.size(2) &&
              (glu ? 2 : 1) * out.size(1) == w.size(1),
              "expert_linear: shapes differ");
  if (src) {
    check(*src, torch::kInt32, "src");
    TORCH_CHECK(src->numel() == out.size(0), "one source per row");
  } else {
    TORCH_CHECK(x.size(0) == out.size(0), "expert_linear: rows differ");
  }
  if (out.size(0) == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    auto a = product<T>(out, x, w);
    a.m = out.size(0);
    a.src = ptr<int>(src); a.start = ptr<int>(start);
    a.tiles = ptr<int>(tiles); a.max_tiles = (tiles.numel() - 1) / 2;
    if (act == "gelu") a.act = Act::GELU;
    if (glu) { a.act = Act::GLU; a.glu = glu_of(act); a.limit = limit; }
    group_gemm(a, tile, "expert_linear");
  });
}

void silu_mul(Tensor out, Tensor x) {
  const int f = out.size(-1);
  TORCH_CHECK(x.size(-1) == 2 * f && x.numel() == 2 * out.numel(),
              "x must be twice as wide as out");
  const long rows = out.numel() / f;
  if (rows == 0) return;
  by_type(x, [&](auto tag) {
    using T = decltype(tag);
    check(x, Scalar<T>::type, "x");
    check(out, Scalar<T>::type, "out");
    if constexpr (std::is_same_v<T, bf16_t>) {
      if (f % 8 == 0) {
        launch_silu_mul(ptr<T>(out), ptr<T>(x), rows, f, stream());
        return;
      }
    }
    launch_silu_mul_any(ptr<T>(out), ptr<T>(x), rows, f, stream());
  });
  post("silu_mul");
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("stream_norm", &stream_norm);
  m.def("embed_norm", &embed_norm);
  m.def("qkv_prepare", &qkv_prepare);
  m.def("attn_ctx", &attn_ctx);
  m.def("silu_mul", &silu_mul);
  m.def("attn_flat", &attn_flat);
  m.def("latent_gather", &latent_gather);
  m.def("latent_prepare", &latent_prepare);
  m.def("head_linear", &head_linear);
  m.def("router_scores", &router_scores);
  m.def("side_gate", &side_gate);
  m.def("moe_select", &moe_select, py::arg("ids"), py::arg("weights"),
        py::arg("z"), py::arg("groups"), py::arg("keep"),
        py::arg("bias") = py::none(), py::arg("over_chosen") = false,
        py::arg("sigmoid") = false, py::arg("correction") = py::none(),
        py::arg("group_best") = 1);
  m.def("moe_tile", &moe_tile);
  m.def("moe_sort", &moe_sort);
  m.def("expert_linear", &expert_linear);
  m.def("linear32", &linear32);
  bind_mixers(m);
}
