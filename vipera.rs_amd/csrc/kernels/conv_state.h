// What a short causal convolution over time keeps between two steps of a request: its inputs of the last taps - 1 tokens, in
// the request's state row.
#pragma once
#include "common.h"

namespace {
// The convolution's inputs of an entry's last taps - 1 tokens become the state; runs after the convolution has read
// the old rows.  Grid (entries, ceil(C / 256)), a thread per channel.
__global__ __launch_bounds__(256) void conv_keep_kernel(const float* __restrict__ in, long long ldi, int taps, int C,
                                                        float* __restrict__ state, long long state_stride,
                                                        long long conv_offset, const int* __restrict__ entry_start,
                                                        const int* __restrict__ entry_first,
                                                        const int* __restrict__ slots) {
  const int e = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int start = entry_start[e], count = entry_start[e + 1] - start;
  if (count <= 0) return;
  const bool fresh = entry_first[e] == 0;
  float* rows = state + (long long)slots[e] * state_stride + conv_offset;
  const int keep = taps - 1;
  for (int j = 0; j < keep; ++j) {           // ascending: row j + count is read before it is written
    const int from = j + count;              // index into [old rows (keep) | the entry's tokens (count)]
    const bool in_step = from >= keep;
    const float* source = in_step ? in + (long long)(start + from - keep) * ldi + c : rows + (long long)from * C + c;
    const float x = *source;
    rows[(long long)j * C + c] = (in_step || !fresh) ? x : 0.f;
  }
}
}  // namespace
