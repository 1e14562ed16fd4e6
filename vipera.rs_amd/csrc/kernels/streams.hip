// Several residual streams per token (hyper-connections), and norms with a mean.
//
// A model with `S` streams keeps x_1 .. x_S per token instead of one residual.  A sublayer reads
// u = sum_s read[s] x_s through its norm and gives y; then x_t <- sum_s mix[s, t] x_s + share[t] y, all streams at once
// from the old ones.  One kernel does the end of one sublayer and the beginning of the next: it takes the old streams
// and y, makes the new streams, writes them, sums them with the next sublayer's weights and norms the sum, so the
// streams are read and written once per sublayer.  All of it is 32-bit.
#include "common.h"

namespace {
typedef float sf4 __attribute__((ext_vector_type(4)));

struct StreamsStep {
  const float* src;          // old streams: token t, stream s at src + t * token_stride + s * stream_stride
  long long token_stride;    // (a stream stride of 0: every stream is the same row, as at the start)
  long long stream_stride;
  const float* y;            // [T, W] the sublayer's output, or null: the streams stay as they are
  const float* mix;          // [S, S], from row s to column t
  const float* share;        // [S]
  float* dst;                // [T, S, W] the new streams, or null: not kept; may be `src`
  const float* read;         // [S], or null: ones
  int norm;                  // 0: u as it is, 1: u over its root mean square, 2: mean off, over the standard deviation
  const float* weight;       // [W], or null: ones
  const float* bias;         // [W], or null: zeros
  float eps;
  const int* rows;           // which token each output row is, or null: one row per token
  int S, W;
};

template <int V> struct Cols { float v[V]; };

template <int V> __device__ __forceinline__ Cols<V> cols_load(const float* p) {
  Cols<V> r;
  if constexpr (V == 4) {
    const sf4 x = *(const sf4*)p;
#pragma unroll
    for (int j = 0; j < 4; ++j) r.v[j] = x[j];
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) r.v[j] = p[j];
  }
  return r;
}

template <int V> __device__ __forceinline__ void cols_store(float* p, const Cols<V>& x) {
  if constexpr (V == 4) {
    sf4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = x.v[j];
    *(sf4*)p = o;
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) p[j] = x.v[j];
  }
}

// One workgroup per output row; a thread owns V consecutive columns in each of KEPT places and keeps their u in
// registers across the norm's sums.  Every thread reads its columns of all old streams before it writes one of the new,
// so `dst` may be `src`.  ST: the number of streams, or 0 for any number up to 8.
template <int ST, int V, int KEPT, typename TO>
__global__ __launch_bounds__(256) void streams_step_kernel(StreamsStep a, TO* __restrict__ out) {
  constexpr int N = ST ? ST : 8;
  __shared__ float scratch[16];
  const int S = ST ? ST : a.S, W = a.W;
  const long long r = blockIdx.x;
  const long long t = a.rows ? a.rows[r] : r;
  const float* src = a.src + t * a.token_stride;
  float read[N], share[N], mix[N][N];
#pragma unroll
  for (int s = 0; s < N; ++s) {
    const bool in = s < S;
    read[s] = !in ? 0.f : a.read ? a.read[s] : 1.f;
    share[s] = (in && a.y) ? a.share[s] : 0.f;
#pragma unroll
    for (int q = 0; q < N; ++q) mix[s][q] = (in && q < S && a.y) ? a.mix[s * S + q] : 0.f;
  }
  // Up to EARLY places: everything the row needs is asked for at once, the norm's weights too, ahead of the first use
  // (a step of few tokens is all latency).  A place past the row's end asks for the last columns and drops them.
  constexpr bool EARLY = KEPT <= 4;
  constexpr int XS = EARLY ? KEPT : 1;
  Cols<V> x[XS][N], y[XS], weight[XS], bias[XS];
  auto ask = [&](int i, int at) {
    const int c = min(((int)threadIdx.x + (int)blockDim.x * i) * V, W - V);
#pragma unroll
    for (int s = 0; s < N; ++s)
      if (s < S) x[at][s] = cols_load<V>(src + s * a.stream_stride + c);
    if (a.y) y[at] = cols_load<V>(a.y + t * W + c);
    if constexpr (EARLY) {
      if (a.weight) weight[at] = cols_load<V>(a.weight + c);
      if (a.bias) bias[at] = cols_load<V>(a.bias + c);
    }
  };
  if constexpr (EARLY) {
#pragma unroll
    for (int i = 0; i < KEPT; ++i) ask(i, i);
  }
  Cols<V> u[KEPT];
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < KEPT; ++i) {
    const int c = ((int)threadIdx.x + (int)blockDim.x * i) * V, at = EARLY ? i : 0;
#pragma unroll
    for (int j = 0; j < V; ++j) u[i].v[j] = 0.f;
    if (c >= W) continue;
    if constexpr (!EARLY) ask(i, 0);
    if (a.y) {
      Cols<V> n[N];
#pragma unroll
      for (int q = 0; q < N; ++q) {
        if (q >= S) continue;
#pragma unroll
        for (int j = 0; j < V; ++j) {
          float v = 0.f;
#pragma unroll
          for (int s = 0; s < N; ++s)
            if (s < S) v = fmaf(mix[s][q], x[at][s].v[j], v);
          n[q].v[j] = fmaf(share[q], y[at].v[j], v);
        }
      }
#pragma unroll
      for (int q = 0; q < N; ++q)
        if (q < S) {
          x[at][q] = n[q];
          if (a.dst) cols_store<V>(a.dst + (t * S + q) * W + c, n[q]);
        }
    }
#pragma unroll
    for (int s = 0; s < N; ++s)
      if (s < S) {
#pragma unroll
        for (int j = 0; j < V; ++j) u[i].v[j] = fmaf(read[s], x[at][s].v[j], u[i].v[j]);
      }
#pragma unroll
    for (int j = 0; j < V; ++j) sum += a.norm == 1 ? u[i].v[j] * u[i].v[j] : u[i].v[j];
  }
  if (out == nullptr) return;
  float mean = 0.f, inv = 1.f;
  if (a.norm) {
    sum = block_sum(sum, scratch) / (float)W;
    if (a.norm == 2) {
      mean = sum;
      float dev = 0.f;
#pragma unroll
      for (int i = 0; i < KEPT; ++i) {
        const int c = ((int)threadIdx.x + (int)blockDim.x * i) * V;
        if (c < W) {
#pragma unroll
          for (int j = 0; j < V; ++j) {
            const float d = u[i].v[j] - mean;
            dev = fmaf(d, d, dev);
          }
        }
      }
      sum = block_sum(dev, scratch) / (float)W;
    }
    inv = 1.0f / sqrtf(sum + a.eps);
  }
  TO* dst = out + r * W;
#pragma unroll
  for (int i = 0; i < KEPT; ++i) {
    const int c = ((int)threadIdx.x + (int)blockDim.x * i) * V;
    if (c >= W) continue;
    Cols<V> o;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      o.v[j] = (u[i].v[j] - mean) * inv;
      if (a.weight) o.v[j] *= EARLY ? weight[EARLY ? i : 0].v[j] : a.weight[c + j];
      if (a.bias) o.v[j] += EARLY ? bias[EARLY ? i : 0].v[j] : a.bias[c + j];
    }
    if constexpr (V == 4 && sizeof(TO) == 2) {
      typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
      bf4 b;
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = (__bf16)o.v[j];
      *(bf4*)(dst + c) = b;
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) dst[c + j] = from_float<TO>(o.v[j]);
    }
  }
}

template <int ST, typename TO>
int launch_step(const StreamsStep& a, TO* out, int num_rows, bool vector, hipStream_t s) {
  const int units = vector ? a.W / 4 : a.W;
  const int threads = units >= 256 ? 256 : (units + 63) / 64 * 64;
  const int kept = (units + threads - 1) / threads;
#define VK_STREAMS(V, KEPT) streams_step_kernel<ST, V, KEPT, TO><<<num_rows, threads, 0, s>>>(a, out)
  if (vector) {
    if (kept <= 2) VK_STREAMS(4, 2);
    else if (kept <= 4) VK_STREAMS(4, 4);
    else if (kept <= 16) VK_STREAMS(4, 16);
    else return VK_UNSUPPORTED_SIZE;
  } else {
    if (kept <= 4) VK_STREAMS(1, 4);
    else if (kept <= 8) VK_STREAMS(1, 8);
    else if (kept <= 64) VK_STREAMS(1, 64);
    else return VK_UNSUPPORTED_SIZE;
  }
#undef VK_STREAMS
  VK_LAUNCH_CHECK();
  return 0;
}

template <typename TO> int launch_streams(const StreamsStep& a, TO* out, int num_rows, bool vector, hipStream_t s) {
  switch (a.S) {
    case 1: return launch_step<1, TO>(a, out, num_rows, vector, s);
    case 2: return launch_step<2, TO>(a, out, num_rows, vector, s);
    case 3: return launch_step<3, TO>(a, out, num_rows, vector, s);
    case 4: return launch_step<4, TO>(a, out, num_rows, vector, s);
    default: return launch_step<0, TO>(a, out, num_rows, vector, s);
  }
}
}  // namespace

extern "C" int vk_streams_step(const float* src, long long token_stride, long long stream_stride, const float* y,
                               const float* mix, const float* share, float* dst, const float* read, int norm,
                               const float* weight, const float* bias, float eps, const int* rows, void* out, int out_dtype,
                               int num_rows, int streams, int width, void* stream) {
  if (num_rows <= 0) return 0;
  if (streams < 1 || width < 1 || norm < 0 || norm > 2 || !src || (y && (!mix || !share)) || (dst && (!y || rows)) ||
      (!dst && !out))
    return VK_BAD_ARGUMENT;
  if (streams > 8) return VK_UNSUPPORTED_SIZE;
  const StreamsStep a{src, token_stride, stream_stride, y, mix, share, dst, read, norm, weight, bias, eps, rows, streams, width};
  const bool vector = width % 4 == 0 && token_stride % 4 == 0 && stream_stride % 4 == 0 &&
                      (((uintptr_t)src | (uintptr_t)y | (uintptr_t)dst | (uintptr_t)out | (uintptr_t)weight | (uintptr_t)bias) & 15) == 0;
  hipStream_t s = (hipStream_t)stream;
  if (out == nullptr || out_dtype == DT_F32) return launch_streams<float>(a, (float*)out, num_rows, vector, s);
  if (out_dtype == DT_BF16) return launch_streams<bf16_t>(a, (bf16_t*)out, num_rows, vector, s);
  return VK_BAD_ARGUMENT;
}
