// Work on the heads of an attention layer before and behind the paged attention kernels, and small per-row steps of
// layers whose sublayers are normed behind instead of in front. All arithmetic is 32-bit.
#include "common.h"
#include "conv_state.h"

namespace {
constexpr int HEAD_REGS = 4;   // a lane keeps up to four numbers of a head: heads of up to 256 numbers

// ---------------------------------------------------------------------------------------------
// head_prepare: the 32-bit sums of a [q | k | v] product become the rows that the rotation-free cache write and the
// attention kernels read, every head at one padded width W.
//   proj [T, ldp]: q (heads * maps * dim) | k (kv_heads * maps * dim) | v (kv_heads * vdim) from column 0 on
//   rotation   the first rot_dims numbers of a q or k head in the half-split layout: pair (i, i + rot_dims / 2) turns
//              by float(position) * inv_freq[i], sine and cosine times `amplitude`; rot_dims 0: none
//   norm       0 none; 1 every q and k head divided by its root mean square (eps inside the root) and multiplied by a
//              weight of `dim` numbers shared by the heads (null: no weight); norm_first: before the rotation, else
//              behind it
//   maps       1, or m attention maps per head: a query head's m maps lie one behind the other in proj and become m
//              query heads, map j in columns [j dim, (j + 1) dim) of its padded head and zeros elsewhere; a key head's
//              m maps stay side by side as one key head of m dim numbers. Query (h, j) then meets exactly map j of its
//              key head, and all maps of a head read the same values.
//   qkv  [T, (heads * maps + 2 kv_heads) * W], W >= max(maps * dim, vdim)
//   k_cache [page, kv_head, slot, W], v_cache [page, kv_head, W, slot] (transposed), or null: the tokens' key and
//   value heads, as they stand in qkv, also go into their pages (page of position p = table[entry, p / block_size]; a
//   negative page id writes nothing), which saves the launch that would only copy them there
// One wave per (token, source head): heads * maps + kv_heads * maps + kv_heads of them a token.
template <typename TO>
__global__ __launch_bounds__(256) void head_prepare_kernel(
    const float* __restrict__ proj, long long ldp, const float* __restrict__ q_weight, const float* __restrict__ k_weight,
    int norm, int norm_first, float eps, const int* __restrict__ positions, const float* __restrict__ inv_freq,
    int rot_dims, float amplitude, int heads, int kv_heads, int maps, int dim, int vdim, int W, long long units,
    TO* __restrict__ qkv,
    TO* __restrict__ k_cache, TO* __restrict__ v_cache, const int* __restrict__ entry_of_token,
    const int* __restrict__ block_table, int table_width, int block_size) {
  const int lane = threadIdx.x & (WAVE - 1);
  const long long unit = (long long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
  if (unit >= units) return;
  const int qk_units = (heads + kv_heads) * maps, all = qk_units + kv_heads;
  const long long t = unit / all;
  const int u = (int)(unit % all);
  const float* src = proj + t * ldp;
  TO* row = qkv + t * (long long)(heads * maps + 2 * kv_heads) * W;
  int page = -1, slot = 0;
  if (k_cache != nullptr && u >= heads * maps) {
    const int pos = positions[t];
    page = block_table[(size_t)entry_of_token[t] * table_width + pos / block_size];
    slot = pos % block_size;
  }
  if (u >= qk_units) {                                   // a value head: copied, padded with zeros
    const int g = u - qk_units;
    const float* x = src + (long long)qk_units * dim + (long long)g * vdim;
    TO* dst = row + (long long)(heads * maps + kv_heads + g) * W;
    TO* paged = page >= 0 ? v_cache + (((size_t)page * kv_heads + g) * W) * block_size + slot : nullptr;
    for (int d = lane; d < W; d += WAVE) {
      const TO v = from_float<TO>(d < vdim ? x[d] : 0.f);
      dst[d] = v;
      if (paged) paged[(size_t)d * block_size] = v;
    }
    return;
  }
  const bool is_q = u < heads * maps;
  const float* x = src + (long long)u * dim;             // q maps and k maps lie one behind the other
  const float* weight = is_q ? q_weight : k_weight;
  const int half = rot_dims / 2;
  float y[HEAD_REGS];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < HEAD_REGS; ++i) {
    const int d = lane + WAVE * i;
    y[i] = d < dim ? x[d] : 0.f;
    ss = fmaf(y[i], y[i], ss);
  }
  float inv = 1.f;
  if (norm && norm_first) {
    inv = 1.0f / sqrtf(wave_sum(ss) / (float)dim + eps);
#pragma unroll
    for (int i = 0; i < HEAD_REGS; ++i) {
      const int d = lane + WAVE * i;
      if (d < dim) y[i] = weight ? y[i] * inv * weight[d] : y[i] * inv;
    }
  }
  if (rot_dims > 0) {
    const float pos = (float)positions[t];
    float partner[HEAD_REGS];
#pragma unroll
    for (int i = 0; i < HEAD_REGS; ++i) {                // the partner's number, normed as this lane's own is
      const int d = lane + WAVE * i;
      const int other = d < half ? d + half : d - half;
      float v = 0.f;
      if (d < rot_dims) {
        v = x[other];
        if (norm && norm_first) v = weight ? v * inv * weight[other] : v * inv;
      }
      partner[i] = v;
    }
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < HEAD_REGS; ++i) {
      const int d = lane + WAVE * i;
      if (d < rot_dims) {
        float sn, cs;
        sincosf(pos * inv_freq[d < half ? d : d - half], &sn, &cs);
        y[i] = amplitude * (d < half ? y[i] * cs - partner[i] * sn : y[i] * cs + partner[i] * sn);
      }
      ss = fmaf(y[i], y[i], ss);
    }
  }
  if (norm && !norm_first) {
    inv = 1.0f / sqrtf(wave_sum(ss) / (float)dim + eps);
#pragma unroll
    for (int i = 0; i < HEAD_REGS; ++i) {
      const int d = lane + WAVE * i;
      if (d < dim) y[i] = weight ? y[i] * inv * weight[d] : y[i] * inv;
    }
  }
  if (is_q) {
    TO* dst = row + (long long)u * W;
    const int at = (u % maps) * dim;
    for (int d = lane; d < W; d += WAVE)
      if (d < at || d >= at + dim) dst[d] = from_float<TO>(0.f);
#pragma unroll
    for (int i = 0; i < HEAD_REGS; ++i) {
      const int d = lane + WAVE * i;
      if (d < dim) dst[at + d] = from_float<TO>(y[i]);
    }
  } else {
    const int ku = u - heads * maps, g = ku / maps, j = ku % maps;
    TO* dst = row + (long long)(heads * maps + g) * W;
    TO* paged = page >= 0 ? k_cache + (((size_t)page * kv_heads + g) * block_size + slot) * W : nullptr;
#pragma unroll
    for (int i = 0; i < HEAD_REGS; ++i) {
      const int d = lane + WAVE * i;
      if (d < dim) {
        const TO v = from_float<TO>(y[i]);
        dst[j * dim + d] = v;
        if (paged) paged[j * dim + d] = v;
      }
    }
    if (j == maps - 1)
      for (int d = maps * dim + lane; d < W; d += WAVE) {
        dst[d] = from_float<TO>(0.f);
        if (paged) paged[d] = from_float<TO>(0.f);
      }
  }
}

// ---------------------------------------------------------------------------------------------
// head_conv_prepare: the same for queries and keys that pass a short causal convolution over time first, and for values
// that may be the (convolved) keys.
//   proj [T, ldp]: q (heads * dim) | k (kv_heads * dim) | v (kv_heads * vdim, where the layer has values of its own)
//   conv [(heads + kv_heads) * dim, taps], the last column is the current token's, or null (no convolution); it runs over q
//              and k, ahead of norm and rotation. Inputs before an entry's first token come from the state row of its slot
//              ((taps - 1) rows of (heads + kv_heads) * dim numbers, oldest first), or are zero for an entry at position 0.
//              `keep`: every entry is one token, and the wave that reads a head's old inputs moves them on; otherwise
//              conv_keep_kernel follows
//   values     the keys as they leave the convolution, or v
//   norm, rotation as in head_prepare with norm_first; `angles` [T, rot_dims / 2]: the step's (sine, cosine), amplitude
//              included, or null: computed here
//   q  [T, heads * W]; k_cache, v_cache as above: keys and values go into their pages and nowhere else
// One wave per (run of TW tokens, head); it keeps the run's last inputs in registers, so that an input is read once (and
// the taps - 1 before the first). K: the taps that stay in registers (fewer are padded with zeros in front), 0: any number,
// read again for every token. A run's values leave as 16-byte pieces where they fill an aligned piece of a page.
template <typename TO> struct ConvHeads {
  const float* proj;
  long long ldp;
  const float* conv;
  int taps;
  float* state;
  long long state_stride;
  int keep;
  const int *entry_of, *entry_start, *entry_first, *slots;
  const float *q_weight, *k_weight;
  int norm;
  float eps;
  const int* positions;
  const float* inv_freq;
  const float2* angles;
  int rot_dims;
  float amplitude;
  int heads, kv_heads, dim, vdim, own_values, W, tokens;
  TO *q, *k_cache, *v_cache;
  const int* table;
  int table_width, block_size;
};

template <typename TO, int R, int K, int TW>
__global__ __launch_bounds__(256) void head_conv_prepare_kernel(ConvHeads<TO> a, long long units) {
  __shared__ float turned[4][TW][R * WAVE];
  const int lane = threadIdx.x & (WAVE - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const long long unit = (long long)blockIdx.x * (blockDim.x / WAVE) + wave;
  if (unit >= units) return;                             // a wave's work is its own: no barrier follows
  const int qk = a.heads + a.kv_heads, per_token = qk + (a.own_values ? a.kv_heads : 0);
  const int u = (int)(unit % per_token);
  const int t0 = (int)(unit / per_token) * TW, count = min(TW, a.tokens - t0);
  const bool is_q = u < a.heads, is_v = u >= qk;
  const int g = is_q ? 0 : is_v ? u - qk : u - a.heads;
  const int n = is_v ? a.vdim : a.dim;
  const long long base = is_v ? (long long)qk * a.dim + (long long)g * a.vdim : (long long)u * a.dim;
  const int C = qk * a.dim, taps = is_v || !a.conv ? 1 : a.taps;
  constexpr int P = K > 1 ? K - 1 : 1;
  // everything the run needs is asked for before anything is used; a token past the step's last repeats it
  int entry[TW], pos[TW];
  float x[TW][R], w[K > 0 ? K : 1][R], norm_weight[R];
  const float* weight = is_q ? a.q_weight : a.k_weight;
#pragma unroll
  for (int i = 0; i < TW; ++i) {
    const int t = min(t0 + i, a.tokens - 1);
    entry[i] = a.entry_of[t];
    pos[i] = a.positions[t];
#pragma unroll
    for (int r = 0; r < R; ++r) x[i][r] = lane + WAVE * r < n ? a.proj[(long long)t * a.ldp + base + lane + WAVE * r] : 0.f;
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = lane + WAVE * r;
    const bool in = d < n;
    if constexpr (K > 0) {
#pragma unroll
      for (int j = 0; j < K; ++j) {
        const int at = j - (K - taps);                   // column of the stored taps
        w[j][r] = !in || at < 0 ? 0.f : a.conv && !is_v ? a.conv[(base + d) * taps + at] : 1.f;
      }
    }
    norm_weight[r] = (in && a.norm && weight && !is_v) ? weight[d] : 1.f;
  }
  int page[TW];
#pragma unroll
  for (int i = 0; i < TW; ++i) page[i] = is_q ? -1 : a.table[(size_t)entry[i] * a.table_width + pos[i] / a.block_size];
  // a channel's input `back` tokens before token i of the run; `back` is at least 1 and below taps
  auto before = [&](int i, int back, int d) -> float {
    const int e = entry[i], t = min(t0 + i, a.tokens - 1), offset = t - a.entry_start[e];
    if (back <= offset) return a.proj[(long long)(t - back) * a.ldp + base + d];
    return a.entry_first[e] == 0 ? 0.f : a.state[(long long)a.slots[e] * a.state_stride + base + (long long)(taps - 1 - (back - offset)) * C + d];
  };
  float y[TW][R];
  if constexpr (K > 0) {
    float past[P][R];
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      if (i == 0 || entry[i] != entry[i > 0 ? i - 1 : 0]) {        // the run's first token, or another entry's
#pragma unroll
        for (int j = 0; j < K - 1; ++j)
#pragma unroll
          for (int r = 0; r < R; ++r) {
            const int d = lane + WAVE * r, back = K - 1 - j;
            past[j][r] = (d < n && back < taps) ? before(i, back, d) : 0.f;
          }
      }
      if (TW == 1 && a.keep && taps > 1) {
        // row j of the state becomes the input taps - 2 - j tokens before this one
        float* old = a.state + (long long)a.slots[entry[i]] * a.state_stride + base;
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
          for (int back = 0; back < K - 1; ++back)
            if (lane + WAVE * r < n && back < taps - 1)
              old[(long long)(taps - 2 - back) * C + lane + WAVE * r] = back ? past[K - 1 - back][r] : x[i][r];
      }
#pragma unroll
      for (int r = 0; r < R; ++r) {
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < K - 1; ++j) sum = fmaf(w[j][r], past[j][r], sum);
        y[i][r] = fmaf(w[K - 1][r], x[i][r], sum);
#pragma unroll
        for (int j = 0; j + 1 < K - 1; ++j) past[j][r] = past[j + 1][r];
        past[P - 1][r] = x[i][r];
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      float* old = a.state + (long long)a.slots[entry[i]] * a.state_stride + base;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int d = lane + WAVE * r;
        y[i][r] = 0.f;
        if (d >= n) continue;
        float sum = 0.f;
        for (int j = 0; j + 1 < taps; ++j) {
          const float v = before(i, taps - 1 - j, d);
          sum = fmaf(a.conv[(base + d) * taps + j], v, sum);
          if (TW == 1 && a.keep && j > 0) old[(long long)(j - 1) * C + d] = v;
        }
        y[i][r] = taps > 1 ? fmaf(a.conv[(base + d) * taps + taps - 1], x[i][r], sum) : x[i][r];
        if (TW == 1 && a.keep && taps > 1) old[(long long)(taps - 2) * C + d] = x[i][r];
      }
    }
  }
  if (is_v || (!is_q && !a.own_values)) {
    // the run's values, transposed: consecutive positions of a number lie side by side in its page
    constexpr int PIECE = 16 / (int)sizeof(TO);
    bool whole = TW % PIECE == 0 && count == TW && pos[0] % TW == 0 && a.block_size % TW == 0 && page[0] >= 0;
#pragma unroll
    for (int i = 1; i < TW; ++i) whole = whole && entry[i] == entry[0];
    if (whole) {
      typedef TO piece_t __attribute__((ext_vector_type(PIECE)));
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int d = lane + WAVE * r;
        if (d >= a.W) continue;
        TO* dst = a.v_cache + (((size_t)page[0] * a.kv_heads + g) * a.W + d) * a.block_size + pos[0] % a.block_size;
#pragma unroll
        for (int p = 0; p < TW / PIECE; ++p) {
          piece_t v;
#pragma unroll
          for (int i = 0; i < PIECE; ++i) v[i] = from_float<TO>(y[(p * PIECE + i) % TW][r]);
          *(piece_t*)(dst + p * PIECE) = v;
        }
      }
    } else {
#pragma unroll
      for (int i = 0; i < TW; ++i) {
        if (i >= count || page[i] < 0) continue;
        TO* dst = a.v_cache + ((size_t)page[i] * a.kv_heads + g) * a.W * a.block_size + pos[i] % a.block_size;
#pragma unroll
        for (int r = 0; r < R; ++r)
          if (lane + WAVE * r < a.W) dst[(size_t)(lane + WAVE * r) * a.block_size] = from_float<TO>(y[i][r]);
      }
    }
    if (is_v) return;
  }
  if (a.norm) {
    float ss[TW];
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      ss[i] = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) ss[i] = fmaf(y[i][r], y[i][r], ss[i]);
    }
#pragma unroll
    for (int off = WAVE / 2; off > 0; off >>= 1)         // the tokens' sums step by step side by side
#pragma unroll
      for (int i = 0; i < TW; ++i) ss[i] += __shfl_xor(ss[i], off, WAVE);
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      const float inv = 1.0f / sqrtf(ss[i] / (float)n + a.eps);
#pragma unroll
      for (int r = 0; r < R; ++r) y[i][r] = y[i][r] * inv * norm_weight[r];
    }
  }
  if (a.rot_dims > 0) {
    const int half = a.rot_dims / 2;
#pragma unroll
    for (int i = 0; i < TW; ++i)
#pragma unroll
      for (int r = 0; r < R; ++r) turned[wave][i][lane + WAVE * r] = y[i][r];
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int d = lane + WAVE * r;
      if (d >= a.rot_dims) continue;
      const int pair = d < half ? d : d - half;
      const float sign = d < half ? -1.f : 1.f;
      const float freq = a.angles ? 0.f : a.inv_freq[pair];
#pragma unroll
      for (int i = 0; i < TW; ++i) {
        const float other = turned[wave][i][d < half ? d + half : d - half];
        float sn, cs;
        if (a.angles) {
          const float2 v = a.angles[(long long)min(t0 + i, a.tokens - 1) * half + pair];
          sn = v.x;
          cs = v.y;
        } else {
          sincosf((float)pos[i] * freq, &sn, &cs);
          sn *= a.amplitude;
          cs *= a.amplitude;
        }
        y[i][r] = y[i][r] * cs + sign * (other * sn);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < TW; ++i) {
    if (i >= count || (!is_q && page[i] < 0)) continue;
    TO* dst = is_q ? a.q + ((long long)(t0 + i) * a.heads + u) * a.W
                   : a.k_cache + (((size_t)page[i] * a.kv_heads + g) * a.block_size + pos[i] % a.block_size) * a.W;
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (lane + WAVE * r < a.W) dst[lane + WAVE * r] = from_float<TO>(y[i][r]);
  }
}

template <typename TO> int launch_head_conv_prepare(const ConvHeads<TO>& a, hipStream_t s) {
  const int per_token = a.heads + a.kv_heads * (a.own_values ? 2 : 1);
  const bool runs = a.tokens >= 512;          // enough tokens that waves of eight of them still fill the GPU
  const long long units = (long long)(runs ? (a.tokens + 7) / 8 : a.tokens) * per_token;
  const long long blocks = (units + 3) / 4;
  if (blocks > 0x7fffffffLL) return VK_UNSUPPORTED_SIZE;
  const bool few_taps = !a.conv || a.taps <= 4, narrow = a.W <= 2 * WAVE;
#define VK_HEADS(R, K, TW) head_conv_prepare_kernel<TO, R, K, TW><<<(unsigned)blocks, 256, 0, s>>>(a, units)
#define VK_HEADS_K(R)                            \
  if (few_taps) {                                \
    if (runs) VK_HEADS(R, 4, 8);                 \
    else VK_HEADS(R, 4, 1);                      \
  } else {                                       \
    if (runs) VK_HEADS(R, 0, 8);                 \
    else VK_HEADS(R, 0, 1);                      \
  }
  if (narrow) {
    VK_HEADS_K(2)
  } else {
    VK_HEADS_K(4)
  }
#undef VK_HEADS_K
#undef VK_HEADS
  VK_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------------------
// head_finish: the attention kernels' output, heads padded to W, becomes the output product's input.
//   attn [T, heads * maps * W]
//   maps 2: o = a_1 - lambda a_2 with the two maps of a head (differential attention); maps 1: o = a
//   unit_norm: o / sqrt(mean(o^2) + eps) over the head's vdim numbers
//   times `factor`
//   gate [T, ldg] 32-bit, null: none; gate_per_head: one number per head (column h), else one per number (column
//   h vdim + d); the gate is act(g) with act as in the activation kernel (2 silu, 4 sigmoid)
//   out [T, heads * vdim]
// One wave per (token, head).
__device__ __forceinline__ float gate_act(float z, int act) {
  switch (act) {
    case 2: return z / (1.0f + expf(-z));
    case 4: return 1.0f / (1.0f + expf(-z));
    default: return z;
  }
}

template <typename T>
__global__ __launch_bounds__(256) void head_finish_kernel(const T* __restrict__ attn, int maps, float lambda, int unit_norm,
                                                          float eps, float factor, const float* __restrict__ gate,
                                                          long long ldg, int gate_per_head, int act, int heads, int vdim,
                                                          int W, long long units, T* __restrict__ out) {
  const int lane = threadIdx.x & (WAVE - 1);
  const long long unit = (long long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
  if (unit >= units) return;
  const long long t = unit / heads;
  const int h = (int)(unit % heads);
  const T* a = attn + (t * heads + h) * (long long)maps * W;
  float o[HEAD_REGS];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < HEAD_REGS; ++i) {
    const int d = lane + WAVE * i;
    float v = 0.f;
    if (d < vdim) {
      v = to_float<T>(a[d]);
      if (maps == 2) v -= lambda * to_float<T>(a[W + d]);
    }
    o[i] = v;
    ss = fmaf(v, v, ss);
  }
  float mult = factor;
  if (unit_norm) mult *= 1.0f / sqrtf(wave_sum(ss) / (float)vdim + eps);
  if (gate && gate_per_head) mult *= gate_act(gate[t * ldg + h], act);
#pragma unroll
  for (int i = 0; i < HEAD_REGS; ++i) {
    const int d = lane + WAVE * i;
    if (d >= vdim) continue;
    float v = o[i] * mult;
    if (gate && !gate_per_head) v *= gate_act(gate[t * ldg + (long long)h * vdim + d], act);
    out[(t * heads + h) * (long long)vdim + d] = from_float<T>(v);
  }
}

// ---------------------------------------------------------------------------------------------
// rotate_scale: heads of 32-bit numbers rotated in place by their token's position (half-split layout over the first
// rot_dims numbers of a head) and multiplied by `factor`.  x [T, ld], `heads` heads of `dim` numbers from column 0 on.
__global__ void rotate_scale_kernel(float* __restrict__ x, long long ld, const int* __restrict__ positions,
                                    const float* __restrict__ inv_freq, int rot_dims, int heads, int dim, float factor,
                                    long long total) {
  // a thread owns one pair (or, past the rotated numbers, one number)
  const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const int half = rot_dims / 2, per_head = dim - half;
  const long long t = idx / ((long long)heads * per_head);
  const int rest = (int)(idx % ((long long)heads * per_head)), h = rest / per_head, i = rest % per_head;
  float* head = x + t * ld + (long long)h * dim;
  if (i < half) {
    float sn, cs;
    sincosf((float)positions[t] * inv_freq[i], &sn, &cs);
    const float u = head[i], v = head[i + half];
    head[i] = (u * cs - v * sn) * factor;
    head[i + half] = (v * cs + u * sn) * factor;
  } else {
    head[i + half] *= factor;
  }
}

// ---------------------------------------------------------------------------------------------
// row_gate_add: out[r, :] (+)= act(g[r]) * y[r, :], one learned number per row (a sublayer's output gated per token).
__global__ void row_gate_add_kernel(const float* __restrict__ y, const float* __restrict__ g, long long ldg, int act,
                                    float* __restrict__ out, int width, long long total, int accumulate) {
  const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const float v = gate_act(g[(idx / width) * ldg], act) * y[idx];
  out[idx] = accumulate ? out[idx] + v : v;
}
}  // namespace

extern "C" int vk_head_prepare(const float* proj, long long ldp, const float* q_weight, const float* k_weight, int norm,
                               int norm_first, float eps, const int* positions, const float* inv_freq, int rot_dims,
                               float amplitude, int num_tokens, int heads, int kv_heads, int maps, int dim, int vdim, int W, void* qkv,
                               int dtype, void* k_cache, void* v_cache, const int* entry_of_token, const int* block_table,
                               int table_width, int block_size, void* stream) {
  if (num_tokens <= 0) return 0;
  if (k_cache && (!v_cache || !entry_of_token || !block_table || !positions || table_width <= 0 || block_size <= 0))
    return VK_BAD_ARGUMENT;
  if (heads < 1 || kv_heads < 1 || maps < 1 || dim < 1 || vdim < 1 || W < maps * dim || W < vdim) return VK_BAD_ARGUMENT;
  if (dim > HEAD_REGS * WAVE) return VK_UNSUPPORTED_SIZE;
  if (rot_dims < 0 || rot_dims > dim || (rot_dims & 1) || (rot_dims > 0 && (!positions || !inv_freq))) return VK_BAD_ARGUMENT;
  hipStream_t s = (hipStream_t)stream;
  const long long units = (long long)num_tokens * ((heads + kv_heads) * maps + kv_heads);
  const long long blocks = (units + 3) / 4;
  if (blocks > 0x7fffffffLL) return VK_UNSUPPORTED_SIZE;
  if (dtype == DT_F32)
    head_prepare_kernel<float><<<(unsigned)blocks, 256, 0, s>>>(proj, ldp, q_weight, k_weight, norm, norm_first, eps, positions,
                                                                inv_freq, rot_dims, amplitude, heads, kv_heads, maps, dim, vdim, W, units,
                                                                (float*)qkv, (float*)k_cache, (float*)v_cache, entry_of_token,
                                                                block_table, table_width, block_size);
  else if (dtype == DT_BF16)
    head_prepare_kernel<bf16_t><<<(unsigned)blocks, 256, 0, s>>>(proj, ldp, q_weight, k_weight, norm, norm_first, eps, positions,
                                                                 inv_freq, rot_dims, amplitude, heads, kv_heads, maps, dim, vdim, W, units,
                                                                 (bf16_t*)qkv, (bf16_t*)k_cache, (bf16_t*)v_cache,
                                                                 entry_of_token, block_table, table_width, block_size);
  else
    return VK_BAD_ARGUMENT;
  VK_LAUNCH_CHECK();
  return 0;
}

extern "C" int vk_head_conv_prepare(const float* proj, long long ldp, const float* conv, int taps, float* state,
                                    long long state_stride, const int* entry_of, const int* entry_start, const int* entry_first,
                                    const int* slots, int num_entries, const float* q_weight, const float* k_weight, int norm,
                                    float eps, const int* positions, const float* inv_freq, const float* angles, int rot_dims,
                                    float amplitude, int num_tokens, int heads, int kv_heads, int dim, int vdim, int own_values,
                                    int W, void* q, int dtype, void* k_cache, void* v_cache, const int* block_table,
                                    int table_width, int block_size, void* stream) {
  if (num_tokens <= 0) return 0;
  if (heads < 1 || kv_heads < 1 || dim < 1 || vdim < 1 || W < dim || W < vdim || num_entries < 1 || taps < 1) return VK_BAD_ARGUMENT;
  if (!proj || !q || !k_cache || !v_cache || !entry_of || !entry_start || !entry_first || !slots || !positions || !block_table ||
      table_width <= 0 || block_size <= 0 || (!own_values && vdim != dim) || (conv && taps > 1 && !state))
    return VK_BAD_ARGUMENT;
  if (W > HEAD_REGS * WAVE) return VK_UNSUPPORTED_SIZE;
  if (rot_dims < 0 || rot_dims > dim || (rot_dims & 1) || (rot_dims > 0 && !inv_freq && !angles)) return VK_BAD_ARGUMENT;
  hipStream_t s = (hipStream_t)stream;
  const int keep = num_tokens == num_entries;
#define VK_CONV_HEADS(TO)                                                                                                      \
  launch_head_conv_prepare<TO>(                                                                                                \
      ConvHeads<TO>{proj, ldp, conv, conv ? taps : 1, state, state_stride, keep, entry_of, entry_start, entry_first, slots,    \
                    q_weight, k_weight, norm, eps, positions, inv_freq, (const float2*)angles, rot_dims, amplitude, heads,     \
                    kv_heads, dim, vdim, own_values, W, num_tokens, (TO*)q, (TO*)k_cache, (TO*)v_cache, block_table,           \
                    table_width, block_size},                                                                                  \
      s)
  int status = VK_BAD_ARGUMENT;
  if (dtype == DT_F32) status = VK_CONV_HEADS(float);
  else if (dtype == DT_BF16) status = VK_CONV_HEADS(bf16_t);
#undef VK_CONV_HEADS
  if (status != 0 || !conv || taps == 1) return status;
  // one token per entry and a wave per token: the state has moved on already (a run of eight tokens leaves it to this)
  if (keep && num_tokens < 512) return 0;
  const int channels = (heads + kv_heads) * dim;
  dim3 rows(num_entries, (channels + 255) / 256);
  if (rows.y > 65535) return VK_UNSUPPORTED_SIZE;
  conv_keep_kernel<<<rows, 256, 0, s>>>(proj, ldp, taps, channels, state, state_stride, 0, entry_start, entry_first, slots);
  VK_LAUNCH_CHECK();
  return 0;
}

extern "C" int vk_head_finish(const void* attn, int dtype, int maps, float lambda, int unit_norm, float eps, float factor,
                              const float* gate, long long ldg, int gate_per_head, int act, int num_tokens, int heads,
                              int vdim, int W, void* out, void* stream) {
  if (num_tokens <= 0) return 0;
  if (heads < 1 || vdim < 1 || W < vdim || maps < 1 || maps > 2 || (act != 0 && act != 2 && act != 4)) return VK_BAD_ARGUMENT;
  if (vdim > HEAD_REGS * WAVE) return VK_UNSUPPORTED_SIZE;
  hipStream_t s = (hipStream_t)stream;
  const long long units = (long long)num_tokens * heads;
  const long long blocks = (units + 3) / 4;
  if (blocks > 0x7fffffffLL) return VK_UNSUPPORTED_SIZE;
  if (dtype == DT_F32)
    head_finish_kernel<float><<<(unsigned)blocks, 256, 0, s>>>((const float*)attn, maps, lambda, unit_norm, eps, factor, gate,
                                                               ldg, gate_per_head, act, heads, vdim, W, units, (float*)out);
  else if (dtype == DT_BF16)
    head_finish_kernel<bf16_t><<<(unsigned)blocks, 256, 0, s>>>((const bf16_t*)attn, maps, lambda, unit_norm, eps, factor,
                                                                gate, ldg, gate_per_head, act, heads, vdim, W, units,
                                                                (bf16_t*)out);
  else
    return VK_BAD_ARGUMENT;
  VK_LAUNCH_CHECK();
  return 0;
}

extern "C" int vk_rotate_scale(float* x, long long ld, const int* positions, const float* inv_freq, int rot_dims,
                               int num_tokens, int heads, int dim, float factor, void* stream) {
  if (num_tokens <= 0) return 0;
  if (heads < 1 || dim < 1 || rot_dims < 0 || rot_dims > dim || (rot_dims & 1)) return VK_BAD_ARGUMENT;
  if (rot_dims > 0 && (!positions || !inv_freq)) return VK_BAD_ARGUMENT;
  const long long total = (long long)num_tokens * heads * (dim - rot_dims / 2);
  const long long blocks = (total + 255) / 256;
  if (blocks > 0x7fffffffLL) return VK_UNSUPPORTED_SIZE;
  rotate_scale_kernel<<<(unsigned)blocks, 256, 0, (hipStream_t)stream>>>(x, ld, positions, inv_freq, rot_dims, heads, dim,
                                                                         factor, total);
  VK_LAUNCH_CHECK();
  return 0;
}

extern "C" int vk_row_gate_add(const float* y, const float* g, long long ldg, int act, float* out, int num_rows, int width,
                               int accumulate, void* stream) {
  if (num_rows <= 0) return 0;
  if (width < 1 || (act != 0 && act != 2 && act != 4)) return VK_BAD_ARGUMENT;
  const long long total = (long long)num_rows * width;
  const long long blocks = (total + 255) / 256;
  if (blocks > 0x7fffffffLL) return VK_UNSUPPORTED_SIZE;
  row_gate_add_kernel<<<(unsigned)blocks, 256, 0, (hipStream_t)stream>>>(y, g, ldg, act, out, width, total, accumulate);
  VK_LAUNCH_CHECK();
  return 0;
}
