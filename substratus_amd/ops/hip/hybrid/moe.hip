// Choosing experts and packing tokens by expert.
//
//   select   one wave per token: softmax over all experts, the best groups
//            of neighbours, the best experts of those; all in 32 bits.
//   sort     one workgroup: token rows packed by expert, and every expert's
//            rows cut into tiles for the grouped products. The order of an
//            expert's rows is left to chance: no row's result depends on it,
//            and a token's rows are found again through `at`.
#include "typed.h"

namespace {

// index of the largest value (the lowest such index) over the wave
DEV_INLINE void wave_argmax(float& v, int& i) {
  #pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ov = __shfl_xor(v, off, WAVE);
    const int oi = __shfl_xor(i, off, WAVE);
    if (ov > v || (ov == v && oi < i)) { v = ov; i = oi; }
  }
}

constexpr int SW = 4;           // tokens per workgroup

// PL: experts per lane
template <int PL>
__global__ __launch_bounds__(SW * WAVE)
void moe_select_kernel(int* __restrict__ ids, float* __restrict__ weights,
                       const float* __restrict__ z, int rows, int experts,
                       int top, int groups, int keep) {
  extern __shared__ float s_all[];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const long row = (long)blockIdx.x * SW + wave;
  float* s_z = s_all + wave * experts;          // the token's scores
  const bool live = row < rows;
  float v[PL];
  float mx = -INFINITY;
  #pragma unroll
  for (int i = 0; i < PL; ++i) {
    const int e = lane + i * WAVE;
    v[i] = live && e < experts ? z[row * experts + e] : -INFINITY;
    if (e < experts) s_z[e] = v[i];
    mx = fmaxf(mx, v[i]);
  }
  __syncthreads();
  if (!live) return;
  mx = wave_max(mx);
  float sum = 0.f;
  #pragma unroll
  for (int i = 0; i < PL; ++i)
    if (lane + i * WAVE < experts) sum += expf(v[i] - mx);
  sum = wave_sum(sum);

  if (keep < groups) {
    // best score of each group: lanes take groups in turn
    const int size = experts / groups;
    float gv[PL];
    bool kept[PL];
    #pragma unroll
    for (int i = 0; i < PL; ++i) {
      gv[i] = -INFINITY;
      kept[i] = false;
      const int g = lane + i * WAVE;
      if (g < groups)
        for (int e = 0; e < size; ++e) gv[i] = fmaxf(gv[i], s_z[g * size + e]);
    }
    for (int r = 0; r < keep; ++r) {
      float bv = -INFINITY;
      int bi = 0x7fffffff;
      #pragma unroll
      for (int i = 0; i < PL; ++i) {
        const int g = lane + i * WAVE;
        if (g < groups && !kept[i] && (bi == 0x7fffffff || gv[i] > bv)) {
          bv = gv[i]; bi = g;
        }
      }
      wave_argmax(bv, bi);
      #pragma unroll
      for (int i = 0; i < PL; ++i)
        if (lane + i * WAVE == bi) kept[i] = true;
    }
    // experts of the other groups cannot be chosen
    #pragma unroll
    for (int i = 0; i < PL; ++i) {
      const int e = lane + i * WAVE;
      const int g = e < experts ? e / size : 0;
      unsigned long long any[PL];
      #pragma unroll
      for (int j = 0; j < PL; ++j) any[j] = __ballot(kept[j]);
      bool in = false;
      #pragma unroll
      for (int j = 0; j < PL; ++j)
        if (g / WAVE == j) in = any[j] >> (g % WAVE) & 1;
      if (!in) v[i] = -INFINITY;
    }
  }
  for (int r = 0; r < top; ++r) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    #pragma unroll
    for (int i = 0; i < PL; ++i)
      if (v[i] > bv) { bv = v[i]; bi = lane + i * WAVE; }
    wave_argmax(bv, bi);
    if (lane == 0) {
      // scores that are no numbers choose the first expert, with their weight
      ids[row * top + r] = bi < experts ? bi : 0;
      weights[row * top + r] = expf(bv - mx) / sum;
    }
    #pragma unroll
    for (int i = 0; i < PL; ++i)
      if (lane + i * WAVE == bi) v[i] = -INFINITY;
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

void launch_moe_select(int* ids, float* weights, const float* z, int rows,
                       int experts, int top, int groups, int keep,
                       hipStream_t stream) {
  auto go = [&](auto pl) {
    moe_select_kernel<decltype(pl)::value>
        <<<dim3((rows + SW - 1) / SW), dim3(SW * WAVE),
           SW * experts * sizeof(float), stream>>>(ids, weights, z, rows,
                                                   experts, top, groups, keep);
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
