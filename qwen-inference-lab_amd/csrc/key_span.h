// The keys a row sees, for the kernels that cut one row's keys into parts.
//
// A row at position p sees key j iff j <= p and, with a window w, p - j < w or j < keep (first keys that are kept for
// good).  With kept keys the keys between the two ranges are left out in whole steps of 32: the others are numbered
// without them (a "place": keys below hole0 keep their number, keys from hole1 on come right behind), and a part holds
// P places.  Every step of 32 places then holds at least one visible key.  Without kept keys a place is the key itself.
#pragma once
#include "common.h"

struct KeySpan {
  int ctx, lo, keep;                                       // position + 1, first key of the window, kept keys
  int hole0, hole;                                         // places from hole0 on are `hole` below their keys (0: no hole)
  __device__ __forceinline__ KeySpan(int position, int window, int kept) {
    ctx = position + 1;
    lo = window > 0 ? max(0, ctx - window) : 0;
    keep = kept;
    hole0 = 0; hole = 0;
    if (kept > 0) {
      hole0 = (kept + 31) & ~31;
      hole = max(0, (lo & ~31) - hole0);
    }
  }
  __device__ __forceinline__ int places() const { return ctx - hole; }                       // one past the last place
  __device__ __forceinline__ int first_place() const { return keep > 0 ? 0 : lo; }
  __device__ __forceinline__ int key(int place) const { return place + (place >= hole0 ? hole : 0); }
  __device__ __forceinline__ bool visible(int key) const { return key < ctx && (key >= lo || key < keep); }
};
