// What a layer adds to the stream from its own columns of the per-token side table, for a step of few tokens:
//   g = gelu_tanh(Wgate x) * e          Wgate [dim, width], e: the token's `dim` numbers of the side table's rows
//   y = Wproj g                         Wproj [width, dim]
//   x <- x + y / sqrt(mean(y^2) + eps) * norm
// and, if asked for, the norm in front of the next sublayer applied to the new row (RMS, or layer norm: the mean taken off
// first; its bias may be null).  Weights bfloat16, the stream and everything that is summed 32-bit; x and g are rounded to
// bfloat16 in front of their products, as the separate products read them.
#include "common.h"

namespace {
typedef __bf16 ts_bf16x8 __attribute__((ext_vector_type(8)));
typedef float ts_f32x4 __attribute__((ext_vector_type(4)));
constexpr int TS_THREADS = 1024, TS_WAVES = TS_THREADS / WAVE;

// g [T, D] as bfloat16.  Grid (ceil(D / 16), ceil(T / 16)): a workgroup owns 16 rows of Wgate and 16 tokens, its sixteen waves a
// part of the columns each (v_mfma_f32_16x16x32_bf16, the weight as the first operand), TS_STEPS steps of 32 asked for
// at once; the waves' sums are added in order.
constexpr int TS_STEPS = 4;
__global__ __launch_bounds__(TS_THREADS) void token_side_gate_kernel(const float* __restrict__ x, const __bf16* __restrict__ gate,
                                                                     const float* __restrict__ e, long long lde, int T, int W,
                                                                     int D, __bf16* __restrict__ g) {
  __shared__ ts_f32x4 part[TS_WAVES][WAVE];
  const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE, lr = lane & 15, lg = lane >> 4;
  const int j0 = blockIdx.x * 16, t0 = blockIdx.y * 16;
  const __bf16* w_row = gate + (long long)min(j0 + lr, D - 1) * W;
  const float* x_row = x + (long long)min(t0 + lr, T - 1) * W;
  const int steps = (W + 31) / 32;
  ts_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int s0 = wave * TS_STEPS; s0 < steps; s0 += TS_WAVES * TS_STEPS) {
    ts_bf16x8 w[TS_STEPS];
    ts_f32x4 v[TS_STEPS][2];
#pragma unroll
    for (int i = 0; i < TS_STEPS; ++i) {
      const int k = (s0 + i) * 32 + lg * 8;
      const bool in = k < W;                         // W is a multiple of 8
      const ts_bf16x8 zero = {};
      const ts_f32x4 none = {0.f, 0.f, 0.f, 0.f};
      w[i] = in ? *(const ts_bf16x8*)(w_row + k) : zero;
      v[i][0] = in ? *(const ts_f32x4*)(x_row + k) : none;
      v[i][1] = in ? *(const ts_f32x4*)(x_row + k + 4) : none;
    }
#pragma unroll
    for (int i = 0; i < TS_STEPS; ++i) {
      ts_bf16x8 b;
#pragma unroll
      for (int j = 0; j < 8; ++j) b[j] = (__bf16)v[i][j >> 2][j & 3];
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[i], b, acc, 0, 0, 0);
    }
  }
  part[wave][lane] = acc;
  __syncthreads();
  if (tid >= 256) return;
  // thread -> (lane, number of its four): row j0 + lg * 4 + i of Wgate, token t0 + lr
  const int from = tid >> 2, i = tid & 3, j = j0 + (from >> 4) * 4 + i, t = t0 + (from & 15);
  float z = 0.f;
#pragma unroll
  for (int q = 0; q < TS_WAVES; ++q) z += ((const float*)&part[q][from])[i];
  if (j >= D || t >= T) return;
  const float act = 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  g[(long long)t * D + j] = (__bf16)(act * e[t * lde + j]);
}

struct TokenSideAdd {
  float* x;                   // [T, W]
  const __bf16 *g, *proj;     // [T, D], [W, D]; D a multiple of 8
  const float* norm;          // [W]
  float eps;
  const float *next_weight, *next_bias;
  float next_eps;
  int next_layer;
  __bf16* next_out;           // [T, W], or null
  int W, D;
};

// The sum over the workgroup's waves, in their order; `scratch` [TS_WAVES] is written once in a launch, so that one
// barrier does.
__device__ __forceinline__ float ts_block_sum(float v, ts_f32x4* scratch) {
  v = wave_sum(v);
  if ((threadIdx.x & (WAVE - 1)) == 0) ((float*)scratch)[threadIdx.x / WAVE] = v;
  __syncthreads();
  ts_f32x4 q[TS_WAVES / 4];
#pragma unroll
  for (int i = 0; i < TS_WAVES / 4; ++i) q[i] = scratch[i];
  float total = 0.f;
#pragma unroll
  for (int i = 0; i < TS_WAVES; ++i) total += q[i >> 2][i & 3];
  return total;
}

// The rest. One workgroup per token; thread c keeps the columns c, c + 1024, ... (KEPT of them) of the row and of the
// weights, asked for at the start; y goes through LDS [W].  A group of `lanes` lanes takes a row of Wproj, each lane eight
// numbers at a time (and, where D is above 512, several times); TS_ROWS rows are asked for at once.
constexpr int TS_ROWS = 8;
template <int KEPT>
__global__ __launch_bounds__(TS_THREADS) void token_side_add_kernel(TokenSideAdd a) {
  __shared__ float ys[KEPT * TS_THREADS];
  __shared__ ts_f32x4 scratch[3][TS_WAVES / 4];
  const int tid = threadIdx.x, lane = tid & (WAVE - 1);
  const long long t = blockIdx.x;
  float* row = a.x + t * a.W;
  float x[KEPT], norm[KEPT], weight[KEPT], bias[KEPT];
#pragma unroll
  for (int i = 0; i < KEPT; ++i) {
    const int c = min(tid + TS_THREADS * i, a.W - 1);
    x[i] = row[c];
    norm[i] = a.norm[c];
    weight[i] = a.next_out ? a.next_weight[c] : 0.f;
    bias[i] = a.next_bias ? a.next_bias[c] : 0.f;
  }
  int lanes = 1;                                     // the power of two that covers D / 8, at most a wave
  while (lanes < WAVE && lanes * 8 < a.D) lanes <<= 1;
  const int sub = lane & (lanes - 1), stride = TS_THREADS / lanes;
  float ss = 0.f;
  for (int r0 = tid / lanes; r0 < a.W; r0 += stride * TS_ROWS) {
    float sum[TS_ROWS] = {};
    for (int d = sub * 8; d < a.D; d += lanes * 8) {
      ts_bf16x8 w[TS_ROWS];
#pragma unroll
      for (int q = 0; q < TS_ROWS; ++q) w[q] = *(const ts_bf16x8*)(a.proj + (long long)min(r0 + q * stride, a.W - 1) * a.D + d);
      const ts_bf16x8 v = *(const ts_bf16x8*)(a.g + t * a.D + d);
#pragma unroll
      for (int q = 0; q < TS_ROWS; ++q)
#pragma unroll
        for (int i = 0; i < 8; ++i) sum[q] = fmaf((float)w[q][i], (float)v[i], sum[q]);
    }
    for (int off = lanes >> 1; off > 0; off >>= 1)
#pragma unroll
      for (int q = 0; q < TS_ROWS; ++q) sum[q] += __shfl_xor(sum[q], off, WAVE);
#pragma unroll
    for (int q = 0; q < TS_ROWS; ++q) {
      const int r = r0 + q * stride;
      if (sub == 0 && r < a.W) {
        ys[r] = sum[q];
        ss = fmaf(sum[q], sum[q], ss);
      }
    }
  }
  const float inv = 1.0f / sqrtf(ts_block_sum(ss, scratch[0]) / (float)a.W + a.eps);   // (its barrier also publishes ys)
  float again = 0.f;
#pragma unroll
  for (int i = 0; i < KEPT; ++i) {
    const int c = tid + TS_THREADS * i;
    if (c >= a.W) continue;
    x[i] += ys[c] * inv * norm[i];
    row[c] = x[i];
    again += a.next_layer ? x[i] : x[i] * x[i];
  }
  if (a.next_out == nullptr) return;
  float mean = 0.f;
  again = ts_block_sum(again, scratch[1]);
  if (a.next_layer) {
    mean = again / (float)a.W;
    again = 0.f;
#pragma unroll
    for (int i = 0; i < KEPT; ++i)
      if (tid + TS_THREADS * i < a.W) again = fmaf(x[i] - mean, x[i] - mean, again);
    again = ts_block_sum(again, scratch[2]);
  }
  const float next_inv = 1.0f / sqrtf(again / (float)a.W + a.next_eps);
#pragma unroll
  for (int i = 0; i < KEPT; ++i)
    if (tid + TS_THREADS * i < a.W) a.next_out[t * a.W + tid + TS_THREADS * i] = (__bf16)((x[i] - mean) * next_inv * weight[i] + bias[i]);
}
}  // namespace

extern "C" int vk_token_side(float* x, const float* e, long long lde, const void* gate, const void* proj, const float* norm,
                             float eps, const float* next_weight, const float* next_bias, float next_eps, int next_layer,
                             void* next_out, void* g, int num_tokens, int width, int dim, void* stream) {
  if (num_tokens <= 0) return 0;
  if (width < 8 || dim < 8 || width % 8 || dim % 8 || (next_out && !next_weight) ||
      (((uintptr_t)x | (uintptr_t)gate | (uintptr_t)proj | (uintptr_t)g) & 15))
    return VK_BAD_ARGUMENT;
  if (width > 8 * TS_THREADS) return VK_UNSUPPORTED_SIZE;
  hipStream_t s = (hipStream_t)stream;
  token_side_gate_kernel<<<dim3((dim + 15) / 16, (num_tokens + 15) / 16), TS_THREADS, 0, s>>>(x, (const __bf16*)gate, e, lde,
                                                                                              num_tokens, width, dim, (__bf16*)g);
  VK_LAUNCH_CHECK();
  const TokenSideAdd add{x, (const __bf16*)g, (const __bf16*)proj, norm, eps, next_weight, next_bias, next_eps, next_layer,
                         (__bf16*)next_out, width, dim};
  if (width <= 2 * TS_THREADS) token_side_add_kernel<2><<<num_tokens, TS_THREADS, 0, s>>>(add);
  else if (width <= 4 * TS_THREADS) token_side_add_kernel<4><<<num_tokens, TS_THREADS, 0, s>>>(add);
  else token_side_add_kernel<8><<<num_tokens, TS_THREADS, 0, s>>>(add);
  VK_LAUNCH_CHECK();
  return 0;
}
