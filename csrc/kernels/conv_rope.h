// Arguments of the convolution + rotation kernels (hybrid.hip), shared with the op bindings.
#pragma once

#include <stdint.h>

namespace mx {

struct ConvRope {
  const void* x;        // [rows, ldx]: q | k | v projections side by side
  int64_t ldx;
  const float* w;       // [taps, C], C = (H + G) D + G E
  int taps;
  const float* cosb;    // [max_pos, rd / 2]
  const float* sinb;
  int rd, H, G, D, E;
  void *q, *k, *v;      // head-major outputs; k / v may be nullptr (decode)
  int64_t qh, qt;       // q strides: head, row
  int64_t kh, kt, vh, vt;
  void *kc, *vc;        // paged caches [blocks, G, block, Dp / Ep], nullptr: none
  int Dp, Ep;
  const int32_t* bt;
  int maxb, block, chunk;  // chunk: positions a query may look back over; position p is kept at row p % chunk
  void* ring;           // [slots, taps, C] projected values by position % taps, nullptr: none
};

}  // namespace mx
