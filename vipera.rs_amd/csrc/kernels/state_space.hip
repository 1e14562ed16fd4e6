// State-space recurrence with one decay per head and token (Mamba-2, state-space duality), and the gated norm behind it.
//
//   a_t = exp(-exp(a_log_h) dt_t),  dt_t = softplus(dtraw_t + dt_bias_h)
//   S <- a_t S + dt_t B_t x_t^T,    y_t = S^T C_t + skip_h x_t          (S is N x P, one per head)
//
// The heads of a group share B and C.  Everything is 32-bit: the state, step sizes, decays and the products too (the
// matrix cores' 32-bit form, whose sums and factors are 32-bit numbers).
//
// Two forms that compute the same recurrence:
//   * token by token (state_space_step_kernel), for entries of a few tokens: the state is read once, updated and
//     written once;
//   * in chunks of 64 tokens (state_space_scores_kernel, state_space_chunk_kernel), for longer portions of prompts: with
//     c_t the sum of exp(a_log) dt over the chunk up to t, a chunk's outputs are
//       y_t = exp(-c_t) S^T C_t + sum over j <= t of exp(c_j - c_t) dt_j (C_t . B_j) x_j + skip x_t
//     and its end state exp(-c_end) S + sum_j exp(c_j - c_end) dt_j B_j x_j^T: matrix products, with every exponential
//     at most 1.  The sums c are kept as two 32-bit numbers each, made from 64-bit sums: a difference of two of them is
//     as exact as the step sizes are, however large the sums grow.
//
// A request's state is one row of a [slots + 1, floats] tensor, head after head, each [P][N rounded up to 4]; an entry
// that starts at position 0 takes it as zeros.  `entry_start`, `entry_first`, `slots` as in scan.hip.
#include "common.h"

namespace {
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int CHUNK = 64;         // tokens of a chunk
constexpr int MAX_STATES = 256;   // N

__device__ __forceinline__ float ss_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float ss_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

struct StateSpace {
  const float* x;        // [T, ld]: head h at column h * P
  const float* b;        // [T, ld]: group g at column g * N
  const float* c;        // [T, ld]
  long long ld;
  const float* dt;       // [T, lddt]
  long long lddt;
  const float* dt_bias;  // [H]
  const float* a_log;    // [H]
  const float* skip;     // [H]
  float* state;
  long long state_stride;
  const int* entry_start;
  const int* entry_first;
  const int* slots;
  int heads, groups, P, N;
  float* y;              // [T, H * P]
  float* scores;         // [T, G, CHUNK]: C_t . B_j for the tokens j of t's chunk (chunked form)
};

__host__ __device__ __forceinline__ int padded_states(int N) { return (N + 3) & ~3; }

// Four consecutive numbers of a row of N, zeros past its end.  VEC: rows are 16-byte aligned and N is a multiple of 4.
template <bool VEC> __device__ __forceinline__ f32x4 load4(const float* row, int n, int N) {
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if constexpr (VEC) {
    if (n < N) v = *(const f32x4*)(row + n);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i < N) v[i] = row[n + i];
  }
  return v;
}

// ---------------------------------------------------------------------------------------------
// Token by token.  Grid (entries, heads, parts of P).  `lanes` lanes (a power of two) share a row of the state, four
// numbers each; a thread keeps ROWS rows' shares in registers.  Entries of more than `max_tokens` are left alone.
template <int ROWS, bool VEC>
__global__ __launch_bounds__(256) void state_space_step_kernel(StateSpace a, int lanes, int max_tokens) {
  const int e = blockIdx.x, h = blockIdx.y;
  const int t0 = a.entry_start[e], t1 = a.entry_start[e + 1];
  if (t1 <= t0 || t1 - t0 > max_tokens) return;
  const int P = a.P, N = a.N, Np = padded_states(N);
  const int li = threadIdx.x & (lanes - 1), n0 = li * 4;
  const int per_pass = 256 / lanes;
  const int p0 = blockIdx.z * per_pass * ROWS + threadIdx.x / lanes;
  const bool fresh = a.entry_first[e] == 0;
  float* head = a.state + (long long)a.slots[e] * a.state_stride + (long long)h * P * Np;
  f32x4 s[ROWS];
#pragma unroll
  for (int k = 0; k < ROWS; ++k) {
    const int p = p0 + k * per_pass;
    s[k] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && p < P && n0 < Np) s[k] = *(const f32x4*)(head + (long long)p * Np + n0);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n0 + i >= N) s[k][i] = 0.f;
  }
  const float rate = expf(a.a_log[h]), bias = a.dt_bias[h], skip = a.skip[h];
  const int g = h / (a.heads / a.groups);
  for (int t = t0; t < t1; ++t) {
    const f32x4 b = load4<VEC>(a.b + t * a.ld + (long long)g * N, n0, N);
    const f32x4 c = load4<VEC>(a.c + t * a.ld + (long long)g * N, n0, N);
    float x[ROWS];
#pragma unroll
    for (int k = 0; k < ROWS; ++k) {
      const int p = p0 + k * per_pass;
      x[k] = p < P ? a.x[t * a.ld + (long long)h * P + p] : 0.f;
    }
    const float dt = ss_softplus(a.dt[t * a.lddt + h] + bias);
    const float keep = expf(-rate * dt);
#pragma unroll
    for (int k = 0; k < ROWS; ++k) {
      const float dx = dt * x[k];
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[k][i] = fmaf(keep, s[k][i], dx * b[i]);
        sum = fmaf(s[k][i], c[i], sum);
      }
      for (int off = lanes >> 1; off > 0; off >>= 1) sum += __shfl_xor(sum, off, WAVE);
      const int p = p0 + k * per_pass;
      if (li == 0 && p < P) a.y[((long long)t * a.heads + h) * P + p] = fmaf(skip, x[k], sum);
    }
  }
#pragma unroll
  for (int k = 0; k < ROWS; ++k) {
    const int p = p0 + k * per_pass;
    if (p < P && n0 < Np) *(f32x4*)(head + (long long)p * Np + n0) = s[k];
  }
}

// ---------------------------------------------------------------------------------------------
// 16 x 16 x 4 products in 32-bit.  A lane holds one number of each operand: row (left) or column (right) lane & 15, and
// of the four k of an instruction the one that its quarter lane >> 4 stands for.  Which k that is does not matter as long
// as both operands agree, so a quarter q brings k = 4 q + i to instruction i of four and a lane's four numbers are
// consecutive in memory.  Of the sums a lane holds column lane & 15 of rows 4 (lane >> 4) + i.
__device__ __forceinline__ f32x4 mma4(const f32x4& left, const f32x4& right, f32x4 acc) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(left[i], right[i], acc, 0, 0, 0);
  return acc;
}

// scores[t, g, j] = C_t . B_j for the tokens j <= t of t's chunk (of the four tiles of 16 j, those up to t's own).
// Grid (chunks of the longest entry, entries, groups), a wave per 16 tokens t.
template <bool VEC>
__global__ __launch_bounds__(256) void state_space_scores_kernel(StateSpace a, int min_tokens) {
  const int e = blockIdx.y, g = blockIdx.z;
  const int t0 = a.entry_start[e] + blockIdx.x * CHUNK, t1 = a.entry_start[e + 1];
  if (t1 - a.entry_start[e] < min_tokens || t0 >= t1) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, col = lane & 15, q = lane >> 4;
  const int N = a.N;
  if (t0 + 16 * w >= t1) return;
  const float* crow = a.c + (long long)min(t0 + 16 * w + col, t1 - 1) * a.ld + (long long)g * N;
  const float* brow[4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) brow[jt] = a.b + (long long)min(t0 + 16 * jt + col, t1 - 1) * a.ld + (long long)g * N;
  f32x4 acc[4] = {};
  for (int n = 4 * q; n - 4 * q < N; n += 16) {
    const f32x4 c = load4<VEC>(crow, n, N);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
      if (jt <= w) acc[jt] = mma4(c, load4<VEC>(brow[jt], n, N), acc[jt]);
  }
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt > w) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = t0 + 16 * w + 4 * q + i;
      if (t < t1) a.scores[((long long)t * a.groups + g) * CHUNK + 16 * jt + col] = acc[jt][i];
    }
  }
}

// The chunks of one entry, in order, for one head and 16 of its channels.  Grid (tiles of P, heads, entries), eight
// waves: waves 0 to 3 give the outputs of the chunk's tokens 16 w .. 16 w + 15, waves 4 to 7 carry the state, each its
// tiles of 16 state rows w, w + 4, .. (TPW of them) in registers.  LDS holds the state at the chunk's start, the
// channels' inputs and what the decays give, each twice: while one chunk is worked on, the state waves leave the next
// one's state and inputs and wave 0 its decays in the other half, so a chunk costs one barrier.  What a wave reads from
// memory for the next chunk it asks for as soon as it has used this one's.
//
// Off the diagonal of the chunk's 16-token tiles exp(c_j - c_t) is taken as exp(c_j - c_e) exp(c_e - c_t) with e the last
// token of j's tile: both factors are at most 1, the first is made once per token, the second once per lane and tile.
struct ChunkDecays {
  float c_hi[CHUNK], c_lo[CHUNK], step[CHUNK], from_start[CHUNK];
  __attribute__((aligned(16))) float to_tile[CHUNK];   // dt_j exp(c_j - c_e)
  __attribute__((aligned(16))) float to_end[CHUNK];    // dt_j exp(c_j - c_end)
  float whole;                                         // exp(-c_end)
};

// One wave, a lane per token: step sizes and the running sums of the decays' exponents.
__device__ __forceinline__ void chunk_decays(const StateSpace& a, int t0, int count, int last, int h, float rate, float bias,
                                             ChunkDecays& d) {
  const int lane = threadIdx.x & 63;
  const float dt = lane < count ? ss_softplus(a.dt[(long long)min(t0 + lane, last - 1) * a.lddt + h] + bias) : 0.f;
  double sum = (double)(rate * dt);
#pragma unroll
  for (int off = 1; off < WAVE; off <<= 1) {
    const double before = __shfl_up(sum, off, WAVE);
    if (lane >= off) sum += before;
  }
  const double end = __shfl(sum, WAVE - 1, WAVE), tile_end = __shfl(sum, lane | 15, WAVE);
  const float hi = (float)sum;
  d.c_hi[lane] = hi;
  d.c_lo[lane] = (float)(sum - (double)hi);
  d.step[lane] = dt;
  d.from_start[lane] = expf(-hi);
  d.to_tile[lane] = dt * expf((float)(sum - tile_end));
  d.to_end[lane] = dt * expf((float)(sum - end));
  if (lane == 0) d.whole = expf(-(float)end);
}

template <int TPW, bool VEC>
__global__ __launch_bounds__(512) void state_space_chunk_kernel(StateSpace a, int min_tokens) {
  constexpr int NT = 4 * TPW, NROW = 16 * NT + 4, TROW = CHUNK + 4;
  __shared__ __attribute__((aligned(16))) float s_lds[2][16 * NROW];     // [channel][state]
  __shared__ __attribute__((aligned(16))) float x_lds[2][16 * TROW];     // [channel][token]
  __shared__ ChunkDecays decays[2];
  const int h = blockIdx.y, e = blockIdx.z, p0 = blockIdx.x * 16;
  const int first = a.entry_start[e], last = a.entry_start[e + 1];
  if (last - first < min_tokens || last <= first) return;
  // (the wave's number in a scalar register: the two roles part by a scalar branch, so no wave meets the other's barriers)
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), w = wave & 3;
  const int col = lane & 15, q = lane >> 4;
  const int P = a.P, N = a.N, Np = padded_states(N), g = h / (a.heads / a.groups);
  const bool live = p0 + col < P;
  const float rate = expf(a.a_log[h]), bias = a.dt_bias[h];
  if (wave < 4) {
    // ---- outputs
    const float skip = a.skip[h];
    const float* cbase = a.c + (long long)g * N;
    const float* mbase = a.scores + (long long)g * CHUNK + 4 * q;
    f32x4 c[NT], m[4];
    auto load_c = [&](int t0) {
      const float* row = cbase + (long long)min(t0 + 16 * w + col, last - 1) * a.ld;
#pragma unroll
      for (int k = 0; k < NT; ++k) c[k] = load4<VEC>(row, 16 * k + 4 * q, N);
    };
    auto load_m = [&](int t0) {
      const float* row = mbase + (long long)min(t0 + 16 * w + col, last - 1) * a.groups * CHUNK;
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) m[jt] = jt <= w ? *(const f32x4*)(row + 16 * jt) : f32x4{0.f, 0.f, 0.f, 0.f};
    };
    load_c(first);
    load_m(first);
    if (w == 0) chunk_decays(a, first, min(CHUNK, last - first), last, h, rate, bias, decays[0]);
    __syncthreads();
    int half = 0;
    for (int t0 = first; t0 < last; t0 += CHUNK, half ^= 1) {
      const int count = min(CHUNK, last - t0);
      const ChunkDecays& d = decays[half];
      const float* s = s_lds[half] + col * NROW + 4 * q;
      const float* x = x_lds[half] + col * TROW;
      const int t_own = 16 * w + col;
      const float t_hi = d.c_hi[t_own], t_lo = d.c_lo[t_own];
      // what the state at the chunk's start gives
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < NT; ++k) acc = mma4(c[k], *(const f32x4*)(s + 16 * k), acc);
      const bool more = t0 + CHUNK < last;
      if (more) load_c(t0 + CHUNK);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] *= d.from_start[16 * w + 4 * q + i];
      // the chunk's own tokens
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > w) continue;
        const int j0 = 16 * jt + 4 * q;
        f32x4 left;
        if (jt < w) {
          const float gone = (t_hi - d.c_hi[16 * jt + 15]) + (t_lo - d.c_lo[16 * jt + 15]);
          const float rest = expf(-gone);
          const f32x4 weight = *(const f32x4*)(d.to_tile + j0);
#pragma unroll
          for (int i = 0; i < 4; ++i) left[i] = m[jt][i] * (weight[i] * rest);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int j = j0 + i;
            const float gone = (t_hi - d.c_hi[j]) + (t_lo - d.c_lo[j]);
            left[i] = j <= t_own ? m[jt][i] * (d.step[j] * expf(-gone)) : 0.f;
          }
        }
        acc = mma4(left, *(const f32x4*)(x + j0), acc);
      }
      if (more) load_m(t0 + CHUNK);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * w + 4 * q + i;
        if (t < count && live) a.y[((long long)(t0 + t) * a.heads + h) * P + p0 + col] = fmaf(skip, x[t], acc[i]);
      }
      if (more && w == 0)
        chunk_decays(a, t0 + CHUNK, min(CHUNK, last - t0 - CHUNK), last, h, rate, bias, decays[half ^ 1]);
      __syncthreads();
    }
    return;
  }
  // ---- the state
  const bool fresh = a.entry_first[e] == 0;
  float* srow = a.state + (long long)a.slots[e] * a.state_stride + ((long long)h * P + min(p0 + col, P - 1)) * Np;
  const float* xbase = a.x + (long long)h * P + min(p0 + col, P - 1);
  const int tid = threadIdx.x - 256, x_token = tid >> 4;       // channel col (= tid & 15) of tokens x_token + 16 i
  f32x4 s[TPW], b[TPW][4];
  float x_next[4];
  auto load_x = [&](int t0) {
#pragma unroll
    for (int i = 0; i < 4; ++i) x_next[i] = xbase[(long long)min(t0 + x_token + 16 * i, last - 1) * a.ld];
  };
  auto keep_x = [&](int t0, float* dst) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      dst[col * TROW + x_token + 16 * i] = (t0 + x_token + 16 * i < last && live) ? x_next[i] : 0.f;
  };
  auto load_b = [&](int t0) {
#pragma unroll
    for (int k = 0; k < TPW; ++k) {
      const int n = 16 * (w + 4 * k) + col;
      const float* base = a.b + (long long)g * N + min(n, N - 1);
      if (t0 + CHUNK <= last) {
        const float* row = base + (long long)(t0 + 4 * q) * a.ld;
#pragma unroll
        for (int jt = 0; jt < 4; ++jt)
#pragma unroll
          for (int i = 0; i < 4; ++i) b[k][jt][i] = row[(long long)(16 * jt + i) * a.ld];
      } else {
#pragma unroll
        for (int jt = 0; jt < 4; ++jt)
#pragma unroll
          for (int i = 0; i < 4; ++i) b[k][jt][i] = base[(long long)min(t0 + 16 * jt + 4 * q + i, last - 1) * a.ld];
      }
    }
  };
#pragma unroll
  for (int k = 0; k < TPW; ++k) {
    const int n = 16 * (w + 4 * k) + 4 * q;
    s[k] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && live && n < Np) s[k] = *(const f32x4*)(srow + n);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i >= N) s[k][i] = 0.f;
    *(f32x4*)(s_lds[0] + col * NROW + n) = s[k];
  }
  load_x(first);
  load_b(first);
  keep_x(first, x_lds[0]);
  __syncthreads();
  int half = 0;
  for (int t0 = first; t0 < last; t0 += CHUNK, half ^= 1) {
    const bool more = t0 + CHUNK < last;
    if (more) load_x(t0 + CHUNK);
    const ChunkDecays& d = decays[half];
    const float* x = x_lds[half] + col * TROW + 4 * q;
    f32x4 right[4];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      const f32x4 v = *(const f32x4*)(x + 16 * jt), weight = *(const f32x4*)(d.to_end + 16 * jt + 4 * q);
#pragma unroll
      for (int i = 0; i < 4; ++i) right[jt][i] = v[i] * weight[i];
    }
    const float keep = d.whole;
#pragma unroll
    for (int k = 0; k < TPW; ++k) {
      const int n = 16 * (w + 4 * k);
#pragma unroll
      for (int i = 0; i < 4; ++i) s[k][i] *= keep;
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) s[k] = mma4(b[k][jt], right[jt], s[k]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n + 4 * q + i >= N) s[k][i] = 0.f;      // rows past N: B of the last row stood in for them
      *(f32x4*)(s_lds[half ^ 1] + col * NROW + n + 4 * q) = s[k];
    }
    if (more) {
      load_b(t0 + CHUNK);
      keep_x(t0 + CHUNK, x_lds[half ^ 1]);
    }
    __syncthreads();
  }
  if (live) {
#pragma unroll
    for (int k = 0; k < TPW; ++k) {
      const int n = 16 * (w + 4 * k) + 4 * q;
      if (n < Np) *(f32x4*)(srow + n) = s[k];
    }
  }
}

// ---------------------------------------------------------------------------------------------
// v = y * silu(z); every one of `parts` equal parts of a row over its own root mean square; times the weight.
// Grid (ceil(tokens / tokens a workgroup), parts): a part is taken by blockDim.x threads, V consecutive numbers each
// in KEPT places, which stay in registers across the sum; where one wave is enough for a part a workgroup takes four tokens.
template <int V, int KEPT, typename TO>
__global__ __launch_bounds__(256) void gated_part_norm_kernel(const float* __restrict__ y, const float* __restrict__ z,
                                                              long long ldz, const float* __restrict__ weight, float eps,
                                                              int width, int part, int num_tokens, TO* __restrict__ out) {
  __shared__ float scratch[16];
  typedef float vec __attribute__((ext_vector_type(V)));
  typedef TO outvec __attribute__((ext_vector_type(V)));
  const long long t = (long long)blockIdx.x * blockDim.y + threadIdx.y;
  if (t >= num_tokens) return;          // only whole waves: with several tokens a workgroup there is no barrier
  const int at = blockIdx.y * part;
  const float* ys = y + t * width + at;
  const float* zs = z + t * ldz + at;
  vec v[KEPT];
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < KEPT; ++i) {
    const int c = (threadIdx.x + blockDim.x * i) * V;
#pragma unroll
    for (int j = 0; j < V; ++j) v[i][j] = 0.f;
    if (c < part) {
      const vec a = *(const vec*)(ys + c), b = *(const vec*)(zs + c);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        v[i][j] = a[j] * ss_silu(b[j]);
        sum = fmaf(v[i][j], v[i][j], sum);
      }
    }
  }
  sum = blockDim.y > 1 ? wave_sum(sum) : block_sum(sum, scratch);
  const float inv = 1.0f / sqrtf(sum / (float)part + eps);
  TO* dst = out + t * width + at;
#pragma unroll
  for (int i = 0; i < KEPT; ++i) {
    const int c = (threadIdx.x + blockDim.x * i) * V;
    if (c < part) {
      const vec w = *(const vec*)(weight + at + c);
      outvec o;
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = from_float<TO>(v[i][j] * inv * w[j]);
      *(outvec*)(dst + c) = o;
    }
  }
}

template <typename TO>
int launch_part_norm(const float* y, const float* z, long long ldz, const float* weight, float eps, int width, int part,
                     int parts, int num_tokens, bool vector, TO* out, hipStream_t s) {
  const int units = vector ? part / 4 : part;
  const bool one_wave = units <= 128 && num_tokens >= 64;       // a few tokens spread over more workgroups instead
  const dim3 block = one_wave ? dim3(64, 4) : dim3(units >= 256 ? 256 : (units + 63) / 64 * 64);
  const int kept = (units + (int)block.x - 1) / (int)block.x;
  const dim3 grid((num_tokens + block.y - 1) / block.y, parts);
#define VK_PART(V, KEPT) \
  gated_part_norm_kernel<V, KEPT, TO><<<grid, block, 0, s>>>(y, z, ldz, weight, eps, width, part, num_tokens, out)
  if (vector) {
    if (kept <= 2) VK_PART(4, 2);
    else if (kept <= 16) VK_PART(4, 16);
    else return VK_UNSUPPORTED_SIZE;
  } else {
    if (kept <= 4) VK_PART(1, 4);
    else if (kept <= 64) VK_PART(1, 64);
    else return VK_UNSUPPORTED_SIZE;
  }
#undef VK_PART
  VK_LAUNCH_CHECK();
  return 0;
}
}  // namespace

extern "C" long long vk_state_space_head_floats(int P, int N) { return (long long)P * padded_states(N); }

// `scores` null: token by token, whatever an entry's length.  Otherwise entries of up to `step_tokens` tokens go token by
// token and longer ones in chunks; `max_count` is the longest entry, `min_count` the shortest (a form that no entry
// needs is not launched).
extern "C" int vk_state_space(const float* x, const float* b, const float* c, long long ld, const float* dt, long long lddt,
                              const float* dt_bias, const float* a_log, const float* skip, float* state,
                              long long state_stride, const int* entry_start, const int* entry_first, const int* slots,
                              int num_entries, int heads, int groups, int P, int N, float* y, float* scores, int step_tokens,
                              int min_count, int max_count, void* stream) {
  if (num_entries <= 0) return 0;
  if (heads < 1 || groups < 1 || heads % groups || P < 1 || N < 1 || step_tokens < 0 || max_count < 1 || min_count < 1)
    return VK_BAD_ARGUMENT;
  if (N > MAX_STATES || heads > 65535 || groups > 65535 || num_entries > 65535) return VK_UNSUPPORTED_SIZE;
  if (state_stride < heads * vk_state_space_head_floats(P, N) || (state_stride & 3) || ((uintptr_t)state & 15))
    return VK_BAD_ARGUMENT;
  const StateSpace a{x, b, c, ld, dt, lddt, dt_bias, a_log, skip, state, state_stride, entry_start, entry_first, slots,
                     heads, groups, P, N, y, scores};
  const bool vec = N % 4 == 0 && ld % 4 == 0 && (((uintptr_t)b | (uintptr_t)c) & 15) == 0;
  hipStream_t s = (hipStream_t)stream;
  const int limit = scores ? step_tokens : 0x7fffffff;
  if (min_count <= limit) {
    int lanes = 1;
    while (lanes * 4 < N) lanes *= 2;
    constexpr int ROWS = 4;
    const int per_group = 256 / lanes * ROWS;
    dim3 grid(num_entries, heads, (P + per_group - 1) / per_group);
    if (grid.z > 65535) return VK_UNSUPPORTED_SIZE;
    if (vec) state_space_step_kernel<ROWS, true><<<grid, 256, 0, s>>>(a, lanes, limit);
    else state_space_step_kernel<ROWS, false><<<grid, 256, 0, s>>>(a, lanes, limit);
    VK_LAUNCH_CHECK();
  }
  if (scores && max_count > limit) {
    if ((uintptr_t)scores & 15) return VK_BAD_ARGUMENT;
    dim3 pairs((max_count + CHUNK - 1) / CHUNK, num_entries, groups);
    if (vec) state_space_scores_kernel<true><<<pairs, 256, 0, s>>>(a, limit + 1);
    else state_space_scores_kernel<false><<<pairs, 256, 0, s>>>(a, limit + 1);
    VK_LAUNCH_CHECK();
    dim3 grid((P + 15) / 16, heads, num_entries);
    const int tiles = ((N + 15) / 16 + 3) / 4;
#define VK_CHUNK(TPW)                                                                   \
  if (vec) state_space_chunk_kernel<TPW, true><<<grid, 512, 0, s>>>(a, limit + 1);      \
  else state_space_chunk_kernel<TPW, false><<<grid, 512, 0, s>>>(a, limit + 1)
    switch (tiles) {
      case 1: VK_CHUNK(1); break;
      case 2: VK_CHUNK(2); break;
      case 3: VK_CHUNK(3); break;
      default: VK_CHUNK(4); break;
    }
#undef VK_CHUNK
    VK_LAUNCH_CHECK();
  }
  return 0;
}

extern "C" int vk_gated_part_norm(const float* y, const float* z, long long ldz, const float* weight, float eps, int parts,
                                  int num_tokens, int width, void* out, int out_dtype, void* stream) {
  if (num_tokens <= 0) return 0;
  if (width < 1 || parts < 1 || width % parts || parts > 65535) return VK_BAD_ARGUMENT;
  const int part = width / parts;
  const bool vector = part % 4 == 0 && ldz % 4 == 0 && (((uintptr_t)y | (uintptr_t)z | (uintptr_t)weight | (uintptr_t)out) & 15) == 0;
  hipStream_t s = (hipStream_t)stream;
  if (out_dtype == DT_F32)
    return launch_part_norm<float>(y, z, ldz, weight, eps, width, part, parts, num_tokens, vector, (float*)out, s);
  if (out_dtype == DT_BF16)
    return launch_part_norm<bf16_t>(y, z, ldz, weight, eps, width, part, parts, num_tokens, vector, (bf16_t*)out, s);
  return VK_BAD_ARGUMENT;
}
