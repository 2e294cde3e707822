// What the recurrent kernels share: finding a request's rows in a step, and sums over a row of 16 lanes.
#pragma once
#include "common.h"

// first row and number of rows of request `req` in the ascending list row_req[0 .. n)
__device__ __forceinline__ void rows_of_request(const int* __restrict__ row_req, int n, int req, int& lo, int& cnt) {
  if (req < n) {
    // a step of single rows has request r's one row at place r: three loads side by side in place of two searches.
    // In an ascending list, a place that holds r between two neighbours that do not is all of r's rows.
    const int here = row_req[req];
    const int before = req > 0 ? row_req[req - 1] : -1;
    const int after = req + 1 < n ? row_req[req + 1] : 0x7fffffff;
    if (here == req && before != req && after != req) {
      lo = req;
      cnt = 1;
      return;
    }
  }
  int a = 0, b = n;
  while (a < b) {
    const int mid = (a + b) >> 1;
    if (row_req[mid] < req) a = mid + 1; else b = mid;
  }
  lo = a;
  b = n;
  while (a < b) {
    const int mid = (a + b) >> 1;
    if (row_req[mid] <= req) a = mid + 1; else b = mid;
  }
  cnt = a - lo;
}

__device__ __forceinline__ float row16_sum(float d) {  // over a row of 16 lanes, left in all of them
  d += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, d), 0xB1, 0xF, 0xF, true));
  d += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, d), 0x4E, 0xF, 0xF, true));
  d += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, d), 0x141, 0xF, 0xF, true));
  d += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, d), 0x140, 0xF, 0xF, true));
  return d;
}
