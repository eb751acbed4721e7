// docqa_gate.h -- an output gate in the epilogue of whichever kernel writes the heads
// (DocqaGate, docqa_hybrid.h): sigmoid of columns of a projection, one an element or one a head.
#pragma once
#include "docqa_elem.h"
#include "docqa_hybrid.h"

namespace docqa {

// f[V] *= the gates of elements [c, c + V) of a row's `per`-element groups
template <int V>
__device__ __forceinline__ void apply_gate(const DocqaGate& a, size_t row, int c, float* f) {
  const size_t at = (size_t)(a.row0 + row) * a.ld + a.col;
  float g[V];
  if (a.per == 1) {
    if (a.f32) ld_slabs<V>((const float*)a.P + at + c, a.S, a.slab, g);
    else ld_slabs<V>((const uint16_t*)a.P + at + c, a.S, a.slab, g);
  } else {
    if (a.f32) ld_slabs<1>((const float*)a.P + at + c / a.per, a.S, a.slab, g);
    else ld_slabs<1>((const uint16_t*)a.P + at + c / a.per, a.S, a.slab, g);
#pragma unroll
    for (int j = 1; j < V; ++j) g[j] = g[0];
  }
#pragma unroll
  for (int j = 0; j < V; ++j) f[j] /= 1.f + __expf(-g[j]);
}

}  // namespace docqa

// V-element gates at multiples of V are aligned and lie in one group
static inline bool docqa_gate_vec(const DocqaGate& a, int V) {
  return a.per == 1 ? a.ld % V == 0 && a.col % V == 0 && docqa_aligned16(a.P) : a.per % V == 0;
}
