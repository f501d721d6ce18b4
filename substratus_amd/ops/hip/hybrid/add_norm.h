// Row operations around a 32-bit residual (add_norm.hip).
#pragma once

#include "typed.h"

#include <type_traits>

template <class T>
struct AddNorm {
  T* y;                  // [rows, width]
  float* x;              // [rows, width]
  bool fresh;            // x has nothing to read yet
  const T* rows;         // [rows, width], or null
  const T* pool;         // [any, width], picked by at and wt, or null
  const int* at;         // [rows, picks]
  const float* wt;       // [rows, picks]
  int picks;
  const int* tokens;     // [rows]
  const T* table;        // [vocab, width], or null
  int vocab;
  float scale;
  const float* vec;      // [width], or null
  const float* w;
  const float* b;        // null: RMS norm
  int width;
  float eps;
};

int add_norm_max_width(int width);
template <class T>
void launch_add_norm(const AddNorm<T>&, long rows, hipStream_t);
template <class T>
void launch_joint_gate(T* out, long out_ld, const T* o, const float* w,
                       const T* gate, long g_ld, long rows, int n, float eps,
                       hipStream_t);
template <class T>
void launch_glu(T* out, long out_ld, const T* x, long ld, long rows, int f,
                Glu, float limit, hipStream_t);
template <class T>
void launch_softcap(T* x, long n, float cap, hipStream_t);
