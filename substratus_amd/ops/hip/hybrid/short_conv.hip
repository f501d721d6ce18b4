// Short causal convolutions over time, per channel, for single tokens and
// portions of prompts alike:
//
//   y_t[c] = sum_j weight[c][j] u_(t - taps + 1 + j)[c],  u = x + in_bias
//
// with zeros before a sequence's start. A request's last taps - 1 rows of x
// are its state. A thread has VEC channels of a run of tokens and keeps the
// inputs that later taps need in registers. The thread of a portion's first
// run also leaves the new state: nobody else reads or writes that channel's.
//
//   short_conv   y (+ bias, silu) to rows of their own
//   conv_rope    rows are [q | k]: y of k is the value and goes to its cache;
//                then neighbouring elements of both turn by the row's angles,
//                q to rows of its own, k to its cache
//   conv_qkv     rows are [q | k | v]: q times its position's temperature to
//                rows of its own, k to its cache, v over the root mean square
//                of its head to its cache
#include "short_conv.h"

namespace {

constexpr int BLOCK = 256;
constexpr int RUN = 32;            // tokens per thread

// the first n of VEC channels
template <int VEC, class T>
DEV_INLINE void ld_n(const T* p, int n, float* f) {
  if constexpr (VEC == 4) {
    ldv<4>(p, f);
  } else {
    #pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = j < n ? ld1(p + j) : 0.f;
  }
}

template <int VEC, class T>
DEV_INLINE void st_n(T* p, int n, const float* f) {
  if constexpr (VEC == 4) {
    stv<4>(p, f);
  } else {
    #pragma unroll
    for (int j = 0; j < VEC; ++j)
      if (j < n) st1(p + j, f[j]);
  }
}

// Channels c .. c + n - 1 (n 0: goes along, leaves no state), tokens
// [t0, t0 + run) of entry e;
// emit(row, y, look(row)), where look reads memory ahead of emit's writes.
// TAPS 0: any number, inputs are read again for every tap. ONE: entries have
// one token, for which fewer registers do.
template <int VEC, int TAPS, bool ONE, class T, class L, class F>
DEV_INLINE void convolve(const Conv<T>& a, int e, int c, int n, int t0,
                         int run, L look, F emit) {
  const Entry en = entry_of(a.seq_start, e);
  if (t0 >= en.n) return;
  const int t1 = min(t0 + run, en.n);
  const int taps = TAPS > 0 ? TAPS : a.taps, held = taps - 1;
  const int pos0 = a.positions[en.row0];
  const int slot = a.state_slots[e];
  T* state = slot < 0 ? nullptr
      : a.state + (long)slot * held * a.channels + c;
  const T* x = a.x + (long)en.row0 * a.ld + c;
  float ib[VEC];
  #pragma unroll
  for (int j = 0; j < VEC; ++j) ib[j] = 0.f;
  if (a.in_bias != nullptr) ld_n<VEC>(a.in_bias + c, n, ib);

  // input s (of the entry; below 0: of earlier steps) as it is convolved
  auto input = [&](int s, float* f) {
    if (s >= 0) {
      ld_n<VEC>(x + s * a.ld, n, f);
    } else if (state != nullptr && pos0 + s >= 0) {
      ld_n<VEC>(state + (long)(held + s) * a.channels, n, f);
    } else {
      #pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = 0.f;
      return;
    }
    #pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] += ib[j];
  };

  const float* wp = a.weight + (long)c * taps;
  if constexpr (TAPS > 0) {
    float w[VEC][TAPS], u[TAPS][VEC];
    #pragma unroll
    for (int j = 0; j < VEC; ++j)
      #pragma unroll
      for (int k = 0; k < TAPS; ++k) w[j][k] = j < n ? wp[j * TAPS + k] : 0.f;
    #pragma unroll
    for (int k = 0; k < TAPS - 1; ++k) input(t0 - (TAPS - 1) + k, u[k]);
    auto steps = [&](int t, auto count) {
      constexpr int N = decltype(count)::value;
      float in[N][VEC];
      #pragma unroll
      for (int i = 0; i < N; ++i) input(t + i, in[i]);
      decltype(look(0l)) seen[N];
      #pragma unroll
      for (int i = 0; i < N; ++i) seen[i] = look(en.row0 + t + i);
      #pragma unroll
      for (int i = 0; i < N; ++i) {
        float y[VEC];
        #pragma unroll
        for (int j = 0; j < VEC; ++j) {
          u[TAPS - 1][j] = in[i][j];
          y[j] = 0.f;
          #pragma unroll
          for (int k = 0; k < TAPS; ++k) y[j] += w[j][k] * u[k][j];
          #pragma unroll
          for (int k = 0; k + 1 < TAPS; ++k) u[k][j] = u[k + 1][j];
        }
        emit(en.row0 + t + i, y, seen[i]);
      }
    };
    // tokens at once: fewer if much is looked up for each
    constexpr int AT_ONCE = ONE ? 1 : sizeof(look(0l)) > 4 ? 4 : 8;
    int t = t0;
    if constexpr (!ONE)
      for (; t + AT_ONCE <= t1; t += AT_ONCE)
        steps(t, std::integral_constant<int, AT_ONCE>{});
    for (; t < t1; ++t) steps(t, std::integral_constant<int, 1>{});
  } else {
    for (int t = t0; t < t1; ++t) {
      float y[VEC], f[VEC];
      #pragma unroll
      for (int j = 0; j < VEC; ++j) y[j] = 0.f;
      for (int k = 0; k < taps; ++k) {
        input(t - held + k, f);
        #pragma unroll
        for (int j = 0; j < VEC; ++j)
          if (j < n) y[j] += wp[j * taps + k] * f[j];
      }
      emit(en.row0 + t, y, look(en.row0 + t));
    }
  }
  if (t0 == 0 && state != nullptr && n > 0) {
    // rows move towards the front: each is read before it is written
    for (int k = 0; k < held; ++k) {
      const int s = en.n - held + k;
      float f[VEC];
      #pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = 0.f;
      if (s >= 0) ld_n<VEC>(x + s * a.ld, n, f);
      else if (pos0 + s >= 0)
        ld_n<VEC>(state + (long)(held + s) * a.channels, n, f);
      st_n<VEC>(state + (long)k * a.channels, n, f);
    }
  }
}

template <class T, int VEC, int TAPS, bool ONE>
__global__ __launch_bounds__(BLOCK)
void short_conv_kernel(Conv<T> a, int run) {
  const int c = (blockIdx.x * BLOCK + threadIdx.x) * VEC;
  if (c >= a.channels) return;
  float b[VEC];
  #pragma unroll
  for (int j = 0; j < VEC; ++j) b[j] = 0.f;
  if (a.bias != nullptr) ld_n<VEC>(a.bias + c, VEC, b);
  convolve<VEC, TAPS, ONE>(a, blockIdx.z, c, VEC, blockIdx.y * run, run,
                           [](long) { return 0; },
                           [&](long row, float* y, int) {
    #pragma unroll
    for (int j = 0; j < VEC; ++j) {
      y[j] += b[j];
      if (a.act) y[j] *= sigmoid_f(y[j]);
    }
    st_n<VEC>(a.out + row * a.channels + c, VEC, y);
  });
}

template <class T, int VEC, int TAPS, bool ONE>
__global__ __launch_bounds__(BLOCK)
void conv_rope_kernel(Conv<T> a, int run) {
  const int per = (a.dim + VEC - 1) / VEC, heads = a.channels / a.dim;
  const int i = blockIdx.x * BLOCK + threadIdx.x;
  if (i >= heads * per) return;
  const int head = i / per, d = i % per * VEC;
  // whole pieces of four: launched so
  const int n = VEC == 4 ? 4 : min(VEC, a.dim - d), nq = heads - a.kv;
  const bool key = head >= nq;
  const int pair = d / 2;
  struct Seen {
    int page, at;                      // of the cache
    float turn[VEC];                   // cosine and sine per pair
  };
  convolve<VEC, TAPS, ONE>(a, blockIdx.z, head * a.dim + d, n,
                           blockIdx.y * run, run, [&](long row) {
    Seen f{};
    if (key) {
      const unsigned slot = a.slots[row], size = a.block_size;
      f.page = slot / size;
      f.at = slot % size;
    }
    const float* cs = a.rope + (row * a.half + pair) * 2;
    #pragma unroll
    for (int j = 0; j < VEC; j += 2) {
      const bool there = pair + j / 2 < a.half;
      f.turn[j] = there ? cs[j] : 1.f;
      f.turn[j + 1] = there ? cs[j + 1] : 0.f;
    }
    return f;
  }, [&](long row, float* y, const Seen& f) {
    long at = 0;
    if (key) {
      at = (((long)f.page * a.kv + head - nq) * a.block_size + f.at) * a.dim
           + d;
      st_n<VEC>(a.vc + at, n, y);
    }
    #pragma unroll
    for (int j = 0; j + 1 < VEC; j += 2) {
      const float c = f.turn[j], s = f.turn[j + 1], u = y[j], v = y[j + 1];
      y[j] = u * c - v * s;
      y[j + 1] = v * c + u * s;
    }
    if (key) st_n<VEC>(a.kc + at, n, y);
    else st_n<VEC>(a.q + row * nq * a.dim + head * a.dim + d, n, y);
  });
}

// Place of a row's key or value in the cache.
struct Place {
  int page, at;
};

template <class T>
DEV_INLINE Place place_of(const Conv<T>& a, long row) {
  const unsigned slot = a.slots[row], size = a.block_size;
  return {(int)(slot / size), (int)(slot % size)};
}

// The first nqk workgroups have the queries and keys, VEC elements of a head
// per thread. Every later one has BLOCK / lanes heads of values, whose threads
// (a power of two; more than a wave: the workgroup) sum squares together.
template <class T, int VEC, int TAPS, bool ONE>
__global__ __launch_bounds__(BLOCK)
void conv_qkv_kernel(Conv<T> a, int run, int nqk, int lanes) {
  const int tid = threadIdx.x;
  const int nq = (a.channels - a.kv * (a.dim + a.vdim)) / a.dim;
  if ((int)blockIdx.x < nqk) {
    const int per = (a.dim + VEC - 1) / VEC;
    const int i = blockIdx.x * BLOCK + tid;
    if (i >= (nq + a.kv) * per) return;
    const int head = i / per, d = i % per * VEC;
    const int n = VEC == 4 ? 4 : min(VEC, a.dim - d);
    const bool key = head >= nq;
    struct Seen {
      Place to;
      float f;
    };
    convolve<VEC, TAPS, ONE>(a, blockIdx.z, head * a.dim + d, n,
                             blockIdx.y * run, run, [&](long row) {
      Seen s{{0, 0}, 1.f};
      if (key)
        s.to = place_of(a, row);
      else if (a.temp != 0.f)
        s.f = 1.f + a.temp * log1pf((float)(
            (unsigned)(a.positions[row] + 1) / (unsigned)a.every));
      return s;
    }, [&](long row, float* y, const Seen& s) {
      if (key) {
        st_n<VEC>(a.kc + (((long)s.to.page * a.kv + head - nq) * a.block_size +
                          s.to.at) * a.dim + d, n, y);
      } else {
        #pragma unroll
        for (int j = 0; j < VEC; ++j) y[j] *= s.f;
        st_n<VEC>(a.q + row * nq * a.dim + head * a.dim + d, n, y);
      }
    });
    return;
  }
  __shared__ float s_sum[2][BLOCK / WAVE];
  int turn = 0;
  const int i = (blockIdx.x - nqk) * BLOCK + tid;
  const int head = i / lanes, d = i % lanes * VEC;
  // threads past the end go along: they take part in sums
  const bool mine = head < a.kv && d < a.vdim;
  const int n = !mine ? 0 : VEC == 4 ? 4 : min(VEC, a.vdim - d);
  const int c = (nq + a.kv) * a.dim + (mine ? head * a.vdim + d : 0);
  convolve<VEC, TAPS, ONE>(a, blockIdx.z, c, n, blockIdx.y * run, run,
                           [&](long row) { return place_of(a, row); },
                           [&](long row, float* y, const Place& to) {
    if (a.v_eps >= 0.f) {
      float ss = 0.f;
      #pragma unroll
      for (int j = 0; j < VEC; ++j)
        if (j < n) ss += y[j] * y[j];
      for (int off = 1; off < min(lanes, WAVE); off <<= 1)
        ss += __shfl_xor(ss, off, WAVE);
      if (lanes > WAVE) {
        // two rooms in turn: a token's sums are read before the next but one
        // writes there
        if (tid % WAVE == 0) s_sum[turn][tid / WAVE] = ss;
        __syncthreads();
        ss = 0.f;
        #pragma unroll
        for (int w = 0; w < BLOCK / WAVE; ++w) ss += s_sum[turn][w];
        turn ^= 1;
      }
      const float f = 1.f / sqrtf(ss / (float)a.vdim + a.v_eps);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) y[j] *= f;
    }
    if (mine)
      st_n<VEC>(a.vc + (((long)to.page * a.kv + head) * a.block_size + to.at) *
                       a.vdim + d, n, y);
  });
}

__global__ __launch_bounds__(BLOCK)
void rope_table_kernel(float* __restrict__ out,
                       const int* __restrict__ positions,
                       const double* __restrict__ turns, long rows, int half) {
  const long i = (long)blockIdx.x * BLOCK + threadIdx.x;
  if (i >= rows * half) return;
  double t = (double)positions[i / half] * turns[i % half];
  t -= rint(t);                          // whole turns, before rounding
  float s, c;
  sincospif((float)(2.0 * t), &s, &c);
  out[2 * i] = c;
  out[2 * i + 1] = s;
}

template <class F>
void by_taps(int taps, int max_len, F f) {
  auto go = [&](auto n) {
    if (max_len == 1) f(n, std::true_type{});
    else f(n, std::false_type{});
  };
  switch (taps) {
    case 2: go(std::integral_constant<int, 2>{}); break;
    case 3: go(std::integral_constant<int, 3>{}); break;
    case 4: go(std::integral_constant<int, 4>{}); break;
    default: f(std::integral_constant<int, 0>{}, std::false_type{});
  }
}

template <class T>
bool fours(const Conv<T>& a) {
  return a.channels % 4 == 0 && a.ld % 4 == 0 &&
         reinterpret_cast<uintptr_t>(a.x) % (4 * sizeof(T)) == 0;
}

}  // namespace

// A portion's later runs must not reach back to its state.
static int run_of(int taps, int max_len, long threads) {
  int run = RUN;
  while (run > 8 && threads * ((max_len + run - 1) / run) < 1 << 17) run /= 2;
  return max(run, taps - 1);
}

template <class T>
void launch_short_conv(const Conv<T>& a, int entries, int max_len,
                       hipStream_t stream) {
  auto go = [&](auto vec, auto taps, auto one) {
    constexpr int V = decltype(vec)::value;
    const int units = (a.channels + V - 1) / V;
    const int run = run_of(a.taps, max_len, (long)units * entries);
    short_conv_kernel<T, V, decltype(taps)::value, decltype(one)::value>
        <<<dim3((units + BLOCK - 1) / BLOCK, (max_len + run - 1) / run,
                entries), BLOCK, 0, stream>>>(a, run);
  };
  by_taps(a.taps, max_len, [&](auto taps, auto one) {
    if (fours(a)) go(std::integral_constant<int, 4>{}, taps, one);
    else go(std::integral_constant<int, 1>{}, taps, one);
  });
}

template <class T>
void launch_conv_rope(const Conv<T>& a, int entries, int max_len,
                      hipStream_t stream) {
  auto go = [&](auto vec, auto taps, auto one) {
    constexpr int V = decltype(vec)::value;
    const int units = a.channels / a.dim * ((a.dim + V - 1) / V);
    const int run = run_of(a.taps, max_len, (long)units * entries);
    conv_rope_kernel<T, V, decltype(taps)::value, decltype(one)::value>
        <<<dim3((units + BLOCK - 1) / BLOCK, (max_len + run - 1) / run,
                entries), BLOCK, 0, stream>>>(a, run);
  };
  by_taps(a.taps, max_len, [&](auto taps, auto one) {
    if (fours(a) && a.dim % 4 == 0)
      go(std::integral_constant<int, 4>{}, taps, one);
    else go(std::integral_constant<int, 2>{}, taps, one);
  });
}

// Threads that share a head's values, VEC elements each; more than a wave's
// are a whole workgroup.
static int value_lanes(int vdim, int vec) {
  int lanes = 1;
  while (lanes * vec < vdim) lanes *= 2;
  return lanes > WAVE ? BLOCK : lanes;
}

bool conv_qkv_takes(int vdim) { return vdim <= 2 * BLOCK; }

template <class T>
void launch_conv_qkv(const Conv<T>& a, int entries, int max_len,
                     hipStream_t stream) {
  auto go = [&](auto vec, auto taps, auto one) {
    constexpr int V = decltype(vec)::value;
    const int units = (a.channels - a.kv * a.vdim) / a.dim *
                      ((a.dim + V - 1) / V);
    const int lanes = value_lanes(a.vdim, V);
    const int nqk = (units + BLOCK - 1) / BLOCK;
    const int nv = (a.kv * lanes + BLOCK - 1) / BLOCK;
    const int run = run_of(a.taps, max_len,
                           (long)(units + a.kv * lanes) * entries);
    conv_qkv_kernel<T, V, decltype(taps)::value, decltype(one)::value>
        <<<dim3(nqk + nv, (max_len + run - 1) / run, entries), BLOCK, 0,
           stream>>>(a, run, nqk, lanes);
  };
  by_taps(a.taps, max_len, [&](auto taps, auto one) {
    if (fours(a) && a.dim % 4 == 0 && a.vdim % 4 == 0)
      go(std::integral_constant<int, 4>{}, taps, one);
    else go(std::integral_constant<int, 2>{}, taps, one);
  });
}

void launch_rope_table(float* out, const int* positions, const double* turns,
                       long rows, int half, hipStream_t stream) {
  rope_table_kernel<<<dim3((rows * half + BLOCK - 1) / BLOCK), BLOCK, 0,
                      stream>>>(out, positions, turns, rows, half);
}

#define INSTANTIATE(T)                                                       \
  template void launch_short_conv<T>(const Conv<T>&, int, int, hipStream_t); \
  template void launch_conv_qkv<T>(const Conv<T>&, int, int, hipStream_t);   \
  template void launch_conv_rope<T>(const Conv<T>&, int, int, hipStream_t);
INSTANTIATE(float)
INSTANTIATE(bf16_t)
