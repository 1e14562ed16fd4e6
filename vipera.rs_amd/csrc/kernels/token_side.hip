// What a layer adds to the stream from its own columns of the per-token side table, as one launch for a step of few tokens:
//   g = gelu_tanh(Wgate x) * e          Wgate [dim, width], e: the token's `dim` numbers of the side table's rows
//   y = Wproj g                         Wproj [width, dim]
//   x <- x + y / sqrt(mean(y^2) + eps) * norm
// and, if asked for, the norm in front of the next sublayer applied to the new row (RMS, or layer norm: the mean taken off
// first; its bias may be null).  Weights bfloat16, the stream and everything that is summed 32-bit; x and g are rounded to
// bfloat16 in front of their products, as the separate products read them.
#include "common.h"

namespace {
typedef __bf16 ts_bf16x8 __attribute__((ext_vector_type(8)));
constexpr int TS_THREADS = 1024, TS_WAVES = TS_THREADS / WAVE;

struct TokenSideStep {
  float* x;                   // [T, W]
  const float* e;             // [T, lde], this layer's columns first
  long long lde;
  const __bf16 *gate, *proj;  // [D, W], [W, D]; D and W multiples of 8
  const float* norm;          // [W]
  float eps;
  const float *next_weight, *next_bias;
  float next_eps;
  int next_layer;
  __bf16* next_out;           // [T, W], or null
  int W, D;
};

// One workgroup per token. LDS: x as bfloat16 [W], then y as floats [W], then g [D].
// The gate: a wave per number of g in turn, its lanes along the row; GATES rows are asked for at once.  The projection: a
// group of `lanes` lanes per row of Wproj, each along a part of it.
__global__ __launch_bounds__(TS_THREADS) void token_side_kernel(TokenSideStep a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
  __bf16* xs = (__bf16*)lds;
  float* ys = (float*)(lds + (size_t)a.W * 2);
  float* gs = ys + a.W;
  __shared__ float scratch[16];
  const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE;
  const long long t = blockIdx.x;
  float* x = a.x + t * a.W;
  for (int c = tid; c < a.W; c += TS_THREADS) xs[c] = (__bf16)x[c];
  __syncthreads();
  constexpr int GATES = 4;
  for (int j0 = wave * GATES; j0 < a.D; j0 += TS_WAVES * GATES) {
    float sum[GATES] = {};
    for (int c = lane * 8; c < a.W; c += WAVE * 8) {
      const ts_bf16x8 v = *(const ts_bf16x8*)(xs + c);
      ts_bf16x8 w[GATES];
#pragma unroll
      for (int q = 0; q < GATES; ++q) w[q] = *(const ts_bf16x8*)(a.gate + (long long)min(j0 + q, a.D - 1) * a.W + c);
#pragma unroll
      for (int q = 0; q < GATES; ++q)
#pragma unroll
        for (int i = 0; i < 8; ++i) sum[q] = fmaf((float)w[q][i], (float)v[i], sum[q]);
    }
#pragma unroll
    for (int q = 0; q < GATES; ++q) {
      const float z = wave_sum(sum[q]);
      if (lane == 0 && j0 + q < a.D) {
        const float act = 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
        gs[j0 + q] = (float)(__bf16)(act * a.e[t * a.lde + j0 + q]);
      }
    }
  }
  __syncthreads();
  // lanes of a row of Wproj: the power of two that covers D / 8, at most a wave
  int lanes = 1;
  while (lanes < WAVE && lanes * 8 < a.D) lanes <<= 1;
  const int per_wave = WAVE / lanes, sub = lane & (lanes - 1);
  float ss = 0.f;
  constexpr int ROWS = 4;
  const int stride = TS_WAVES * per_wave;
  for (int r0 = wave * per_wave + lane / lanes; r0 < a.W; r0 += stride * ROWS) {
    float sum[ROWS] = {};
    for (int d = sub * 8; d < a.D; d += lanes * 8) {
      ts_bf16x8 w[ROWS];
#pragma unroll
      for (int q = 0; q < ROWS; ++q) w[q] = *(const ts_bf16x8*)(a.proj + (long long)min(r0 + q * stride, a.W - 1) * a.D + d);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float g = gs[d + i];
#pragma unroll
        for (int q = 0; q < ROWS; ++q) sum[q] = fmaf((float)w[q][i], g, sum[q]);
      }
    }
#pragma unroll
    for (int q = 0; q < ROWS; ++q) {
      for (int off = lanes >> 1; off > 0; off >>= 1) sum[q] += __shfl_xor(sum[q], off, WAVE);
      const int r = r0 + q * stride;
      if (sub == 0 && r < a.W) {
        ys[r] = sum[q];
        ss = fmaf(sum[q], sum[q], ss);
      }
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)a.W + a.eps);   // (its barriers also publish ys)
  float again = 0.f;
  for (int c = tid; c < a.W; c += TS_THREADS) {
    const float v = x[c] + ys[c] * inv * a.norm[c];
    x[c] = v;
    ys[c] = v;
    again += a.next_layer ? v : v * v;
  }
  if (a.next_out == nullptr) return;
  float mean = 0.f;
  if (a.next_layer) {
    mean = block_sum(again, scratch) / (float)a.W;
    again = 0.f;
    for (int c = tid; c < a.W; c += TS_THREADS) again += (ys[c] - mean) * (ys[c] - mean);
  }
  const float next_inv = 1.0f / sqrtf(block_sum(again, scratch) / (float)a.W + a.next_eps);
  for (int c = tid; c < a.W; c += TS_THREADS)
    a.next_out[t * a.W + c] = (__bf16)((ys[c] - mean) * next_inv * a.next_weight[c] + (a.next_bias ? a.next_bias[c] : 0.f));
}
}  // namespace

extern "C" int vk_token_side(float* x, const float* e, long long lde, const void* gate, const void* proj, const float* norm,
                             float eps, const float* next_weight, const float* next_bias, float next_eps, int next_layer,
                             void* next_out, int num_tokens, int width, int dim, void* stream) {
  if (num_tokens <= 0) return 0;
  if (width < 8 || dim < 8 || width % 8 || dim % 8 || (next_out && !next_weight) || (((uintptr_t)gate | (uintptr_t)proj) & 15))
    return VK_BAD_ARGUMENT;
  const size_t bytes = (size_t)width * 6 + (size_t)dim * 4;
  if (bytes > 144 * 1024) return VK_UNSUPPORTED_SIZE;
  static bool sized = false;
  if (!sized) {
    const hipError_t err = hipFuncSetAttribute((const void*)token_side_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024);
    if (err != hipSuccess) return (int)err;
    sized = true;
  }
  token_side_kernel<<<num_tokens, TS_THREADS, bytes, (hipStream_t)stream>>>(
      TokenSideStep{x, e, lde, (const __bf16*)gate, (const __bf16*)proj, norm, eps, next_weight, next_bias, next_eps, next_layer,
                    (__bf16*)next_out, width, dim});
  VK_LAUNCH_CHECK();
  return 0;
}
