// Choosing experts and packing tokens by expert.
//
//   select   one wave per token: scores (sums of a product's shares of the
//            inner dimension), softmax over all experts, the best groups
//            of neighbours, the best experts of those; all in 32 bits.
//            Or the softmax is over the chosen experts only, or every score
//            is a sigmoid. What is best may go by scores with a correction,
//            a group by the sum of its two best.
//   sort     one workgroup: token rows packed by expert, and every expert's
//            rows cut into tiles for the grouped products. The order of an
//            expert's rows is left to chance: no row's result depends on it,
//            and a token's rows are found again through `at`.
#include "typed.h"

namespace {

constexpr int SW = 4;           // tokens per workgroup

// How many of n values (padded with -inf to fours) come before value v of
// index i, that is, are larger, or equal with a lower index. NaNs come last.
DEV_INLINE int rank_of(const float* s, int n, float v, int i) {
  int r = 0;
  for (int j = 0; j < n; j += 4) {
    const float4 f = *reinterpret_cast<const float4*>(s + j);
    r += f.x > v || (f.x == v && j < i);
    r += f.y > v || (f.y == v && j + 1 < i);
    r += f.z > v || (f.z == v && j + 2 < i);
    r += f.w > v || (f.w == v && j + 3 < i);
  }
  return r;
}

// PL: experts per lane
template <int PL>
__global__ __launch_bounds__(SW * WAVE)
void moe_select_kernel(int* __restrict__ ids, float* __restrict__ weights,
                       const float* __restrict__ z, int splits, int rows,
                       int experts, int top, int groups, int keep,
                       const float* __restrict__ bias, bool over_chosen,
                       bool sigmoid, const float* __restrict__ correction,
                       int group_best) {
  extern __shared__ float4 s_all[];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int pad = (experts + 3) / 4 * 4;
  const long row = min((long)blockIdx.x * SW + wave, (long)rows - 1);
  float* s_z = reinterpret_cast<float*>(s_all) + wave * 2 * pad;
  float* s_g = s_z + pad;                       // best score of each group
  const int size = experts / groups;
  float v[PL], sc[PL];                          // for the choice, as weights
  float mx = -INFINITY;
  // scores that are no numbers: weights are none either, but experts are
  for (int r = lane; r < top; r += WAVE) ids[row * top + r] = 0;
  #pragma unroll
  for (int i = 0; i < PL; ++i) {
    const int e = lane + i * WAVE;
    v[i] = e < experts ? z[row * experts + e] : -INFINITY;
    if (e < experts) {
      #pragma unroll 4
      for (int s = 1; s < splits; ++s)
        v[i] += z[((long)s * rows + row) * experts + e];
      if (bias != nullptr) v[i] += bias[e];
      if (sigmoid) v[i] = sigmoid_f(v[i]);
    }
    sc[i] = v[i];
    mx = fmaxf(mx, v[i]);
    if (e < experts && correction != nullptr) v[i] += correction[e];
    if (e < pad) s_z[e] = v[i];
  }
  mx = wave_max(mx);
  float sum = 0.f;
  #pragma unroll
  for (int i = 0; i < PL; ++i)
    if (lane + i * WAVE < experts) sum += expf(sc[i] - mx);
  sum = wave_sum(sum);
  __syncthreads();

  if (keep < groups) {
    float g[PL];
    #pragma unroll
    for (int i = 0; i < PL; ++i) {
      g[i] = -INFINITY;
      const int n = lane + i * WAVE;
      if (n < groups)
      {
        float next = -INFINITY;
        for (int e = 0; e < size; ++e) {
          const float s = s_z[n * size + e];
          next = fmaxf(next, fminf(g[i], s));
          g[i] = fmaxf(g[i], s);
        }
        if (group_best > 1 && size > 1) g[i] += next;
      }
      if (n < pad) s_g[n] = g[i];
    }
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < PL; ++i)
      if (lane + i * WAVE < groups &&
          rank_of(s_g, groups, g[i], lane + i * WAVE) >= keep)
        g[i] = INFINITY;                        // marks a group left out
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < PL; ++i)
      if (lane + i * WAVE < groups) s_g[lane + i * WAVE] = g[i];
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < PL; ++i) {
      const int e = lane + i * WAVE;
      if (e < experts && s_g[e / size] == INFINITY) {
        v[i] = -INFINITY;
        s_z[e] = -INFINITY;
      }
    }
    __syncthreads();
  }
  int r[PL];
  float chosen = 0.f;
  #pragma unroll
  for (int i = 0; i < PL; ++i) {
    const int e = lane + i * WAVE;
    r[i] = e < experts ? rank_of(s_z, experts, v[i], e) : top;
    if (r[i] < top) chosen += expf(sc[i] - mx);
  }
  if (over_chosen) sum = wave_sum(chosen);
  #pragma unroll
  for (int i = 0; i < PL; ++i) {
    if (r[i] < top) {
      ids[row * top + r[i]] = lane + i * WAVE;
      weights[row * top + r[i]] =
          sigmoid ? sc[i] : expf(sc[i] - mx) / sum;
    }
  }
}

constexpr int SORT = 1024;      // threads, and most experts

// inclusive sum over the workgroup
DEV_INLINE int scan(int v, int* s) {
  s[threadIdx.x] = v;
  __syncthreads();
  for (int off = 1; off < SORT; off <<= 1) {
    const int add = (int)threadIdx.x >= off ? s[threadIdx.x - off] : 0;
    __syncthreads();
    s[threadIdx.x] += add;
    __syncthreads();
  }
  const int r = s[threadIdx.x];
  __syncthreads();
  return r;
}

__global__ __launch_bounds__(SORT)
void moe_sort_kernel(int* __restrict__ at, int* __restrict__ src,
                     int* __restrict__ start, int* __restrict__ tiles,
                     const int* __restrict__ ids, int n, int top, int experts,
                     int tile) {
  __shared__ int s_n[SORT], s_scan[SORT];
  const int t = threadIdx.x;
  s_n[t] = 0;
  __syncthreads();
  for (int i = t; i < n; i += SORT) atomicAdd(&s_n[ids[i]], 1);
  __syncthreads();
  const int mine = s_n[t];
  const int end = scan(mine, s_scan);
  const int nt = (mine + tile - 1) / tile;
  const int tend = scan(nt, s_scan);
  if (t < experts) start[t + 1] = end;
  if (t == 0) start[0] = 0;
  if (t == SORT - 1) tiles[0] = tend;
  for (int i = 0; i < nt; ++i) {
    tiles[1 + 2 * (tend - nt + i)] = t;
    tiles[2 + 2 * (tend - nt + i)] = end - mine + i * tile;
  }
  s_n[t] = end - mine;
  __syncthreads();
  for (int i = t; i < n; i += SORT) {
    const int p = atomicAdd(&s_n[ids[i]], 1);
    at[i] = p;
    src[p] = i / top;
  }
}

}  // namespace

int moe_max_experts() { return SORT; }

void launch_moe_select(int* ids, float* weights, const float* z, int splits,
                       int rows, int experts, int top, int groups, int keep,
                       const float* bias, bool over_chosen, bool sigmoid,
                       const float* correction, int group_best,
                       hipStream_t stream) {
  auto go = [&](auto pl) {
    moe_select_kernel<decltype(pl)::value>
        <<<dim3((rows + SW - 1) / SW), dim3(SW * WAVE),
           SW * 2 * ((experts + 3) / 4 * 4) * sizeof(float), stream>>>(
            ids, weights, z, splits, rows, experts, top, groups, keep, bias,
            over_chosen, sigmoid, correction, group_best);
  };
  if (experts <= WAVE) go(std::integral_constant<int, 1>{});
  else if (experts <= 4 * WAVE) go(std::integral_constant<int, 4>{});
  else go(std::integral_constant<int, SORT / WAVE>{});
}

void launch_moe_sort(int* at, int* src, int* start, int* tiles, const int* ids,
                     int n, int top, int experts, int tile,
                     hipStream_t stream) {
  moe_sort_kernel<<<1, SORT, 0, stream>>>(at, src, start, tiles, ids, n, top,
                                          experts, tile);
}
