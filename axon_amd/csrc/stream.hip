// Passes over the 32-bit residual stream that a layer's arrangement asks for:
//   * the embedding with a table of token pairs: x = embed[token] scale + pairs[(previous mul_prev + token mul_cur) mod
//     buckets] (a request's first token: row `buckets`), the previous token being part of a request's state;
//   * the sum: x += sum_j n_j(y_j) s_j over one or two sublayer outputs y_j (32-bit rows), s_j a number a column (a layer
//     scale, the residual's factor, the share of a side), n_j nothing or x / sqrt(mean(x^2) + eps); and, if asked for, the
//     RMS norm of the new row, in steps of single tokens also shifted towards the token before;
//   * the RMS norm with a token shift: h = norm(x), out = h + (h' - h) share, h' the previous token's h (zeros before a
//     request's first), the last h being part of a request's state.
//
// States hold two copies, the one behind position p in copy p & 1 (see recurrence.h).  A step of several tokens of a
// request may end in the copy that it started from: the block of a request's first token in the step therefore reads what
// was kept and then writes what is kept next, every thread its own columns, and no other block touches either.
#include <math.h>

#include "api.h"
#include "common.h"
#include "recurrence.h"

namespace {

#define ST_THREADS 256

// The last token of the request whose token t is: a request's tokens lie side by side.
__device__ inline int last_of_request(const int32_t* __restrict__ seq_rows, int t, int n_tokens) {
  const int slot = seq_rows[t];
  if (t + 1 >= n_tokens || seq_rows[t + 1] != slot) return t;
  int in = t + 1, out = n_tokens;              // `in` belongs to the request, `out` does not
  while (out - in > 1) {
    const int mid = in + (out - in) / 2;
    if (seq_rows[mid] == slot) in = mid; else out = mid;
  }
  return in;
}

__global__ void __launch_bounds__(ST_THREADS)
embed_pairs_kernel(const int32_t* __restrict__ tokens, const elem_t* __restrict__ table, int packed, float scale,
                   const elem_t* __restrict__ pairs, int buckets, long mul_prev, long mul_cur, int32_t* __restrict__ state,
                   const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_rows, float* __restrict__ x, int n_tokens,
                   int dim) {
  __shared__ int pair_row;
  const int t = blockIdx.x, token = tokens[t];
  if (threadIdx.x == 0) {
    const int slot = seq_rows[t], pos = positions[t];
    int before = -1;
    if (t > 0 && seq_rows[t - 1] == slot) {
      before = tokens[t - 1];
    } else {
      if (pos > 0) before = state[2L * slot + ((pos + 1) & 1)];
      const int last = last_of_request(seq_rows, t, n_tokens);
      state[2L * slot + (positions[last] & 1)] = tokens[last];
    }
    pair_row = before < 0 ? buckets : (int)((before * mul_prev + token * mul_cur) % buckets);
  }
  __syncthreads();
  const elem_t* pair = pairs + (size_t)pair_row * dim;
  float* dst = x + (size_t)t * dim;
  if (packed) {
    const elem_t* tile = table + (size_t)(token / 16) * (dim / 32) * 512 + (token % 16) * 8;
    for (int i = threadIdx.x; i < dim; i += ST_THREADS)
      dst[i] = fmaf(to_float(tile[(size_t)(i / 32) * 512 + ((i % 32) / 8) * 128 + i % 8]), scale, to_float(pair[i]));
    return;
  }
  const elem_t* row = table + (size_t)token * dim;
  for (int i = threadIdx.x; i < dim; i += ST_THREADS) dst[i] = fmaf(to_float(row[i]), scale, to_float(pair[i]));
}

// G neighbouring numbers (4 where the width and the addresses allow, else 1).
template <int G>
__device__ inline void st_load(const float* __restrict__ p, float (&v)[G]) {
  if (G == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    v[0] = q.x; v[1 % G] = q.y; v[2 % G] = q.z; v[3 % G] = q.w;
  } else {
    v[0] = p[0];
  }
}
template <int G>
__device__ inline void st_store(float* p, const float (&v)[G]) {
  if (G == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1 % G], v[2 % G], v[3 % G]);
  else p[0] = v[0];
}
template <int G>
__device__ inline void st_store_elem(elem_t* p, const float (&v)[G]) {
#if AXON_BF16
  if (G == 4) *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(v[0], v[1 % G]), pack2_bf16(v[2 % G], v[3 % G]));
  else p[0] = from_float(v[0]);
#else
  st_store<G>(p, v);
#endif
}

// 1 / sqrt(mean(row^2) + eps): a chain a thread, a butterfly a wave, the four waves in order.
template <int G>
__device__ inline float inverse_rms(const float* __restrict__ row, int dim, float eps, float* partial) {
  float ss = 0.0f;
  for (int i = G * threadIdx.x; i < dim; i += G * ST_THREADS) {
    float v[G];
    st_load<G>(row + i, v);
#pragma unroll
    for (int e = 0; e < G; ++e) ss = fmaf(v[e], v[e], ss);
  }
  return 1.0f / sqrtf(block_sum_256(ss, partial) / (float)dim + eps);
}

// A block a row.  y1 may be null; scales are float32 [dim]; norm_eps < 0: that output is taken as it is.  h null: no
// norm behind the sum; share null: no shift.  With a shift every row is a request of its own.
template <int G>
__global__ void __launch_bounds__(ST_THREADS)
scaled_sum_kernel(const float* __restrict__ y0, const float* __restrict__ s0, float norm_eps0, const float* __restrict__ y1,
                  const float* __restrict__ s1, float norm_eps1, float* __restrict__ x, const float* __restrict__ gain, float eps,
                  elem_t* __restrict__ h, const float* __restrict__ share, float* __restrict__ state, long state_stride,
                  const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_rows, int dim) {
  __shared__ float partial[3][ST_THREADS / AXON_WAVE];
  const int t = blockIdx.x;
  const size_t at = (size_t)t * dim;
  const float inv0 = norm_eps0 >= 0.0f ? inverse_rms<G>(y0 + at, dim, norm_eps0, partial[0]) : 1.0f;
  const float inv1 = y1 != nullptr && norm_eps1 >= 0.0f ? inverse_rms<G>(y1 + at, dim, norm_eps1, partial[1]) : 1.0f;
  float ss = 0.0f;
  for (int i = G * threadIdx.x; i < dim; i += G * ST_THREADS) {
    float v[G], y[G], s[G];
    st_load<G>(x + at + i, v);
    st_load<G>(y0 + at + i, y);
    st_load<G>(s0 + i, s);
#pragma unroll
    for (int e = 0; e < G; ++e) y[e] = (y[e] * inv0) * s[e];
    if (y1 != nullptr) {
      float z[G];
      st_load<G>(y1 + at + i, z);
      st_load<G>(s1 + i, s);
#pragma unroll
      for (int e = 0; e < G; ++e) y[e] = fmaf(z[e] * inv1, s[e], y[e]);
    }
#pragma unroll
    for (int e = 0; e < G; ++e) { v[e] += y[e]; ss = fmaf(v[e], v[e], ss); }
    st_store<G>(x + at + i, v);
  }
  if (h == nullptr) return;
  const float inv = 1.0f / sqrtf(block_sum_256(ss, partial[2]) / (float)dim + eps);
  const float* kept = nullptr;
  float* keep = nullptr;
  if (share != nullptr) {
    kept = rec_copy_before(state, state_stride, dim, seq_rows[t], positions[t]);
    keep = rec_copy_behind(state, state_stride, dim, seq_rows[t], positions[t]);
  }
  for (int i = G * threadIdx.x; i < dim; i += G * ST_THREADS) {
    float v[G], g[G];
    st_load<G>(x + at + i, v);                     // what this thread stored above
    st_load<G>(gain + i, g);
#pragma unroll
    for (int e = 0; e < G; ++e) v[e] = (v[e] * inv) * g[e];
    if (share != nullptr) {
      float p[G], m[G];
      st_load<G>(kept + i, p);
      st_load<G>(share + i, m);
      st_store<G>(keep + i, v);
#pragma unroll
      for (int e = 0; e < G; ++e) v[e] = fmaf(p[e] - v[e], m[e], v[e]);
    }
    st_store_elem<G>(h + at + i, v);
  }
}

// A block `run` tokens in a row.
template <int G>
__global__ void __launch_bounds__(ST_THREADS)
shifted_norm_kernel(const float* __restrict__ x, const float* __restrict__ gain, float eps, const float* __restrict__ share,
                    float* __restrict__ state, long state_stride, const int32_t* __restrict__ positions,
                    const int32_t* __restrict__ seq_rows, elem_t* __restrict__ out, int n_tokens, int dim, int run) {
  __shared__ float partial[4][ST_THREADS / AXON_WAVE];
  const int t0 = blockIdx.x * run, t1 = min(t0 + run, n_tokens);
  float inv_before = 0.0f;
  for (int t = t0; t < t1; ++t) {
    const int slot = seq_rows[t];
    const bool inside = t > 0 && seq_rows[t - 1] == slot;
    const float* row = x + (size_t)t * dim;
    if (inside && t == t0) inv_before = inverse_rms<G>(row - dim, dim, eps, partial[2]);
    const float inv = inverse_rms<G>(row, dim, eps, partial[t & 1]);
    const int last = inside ? t : last_of_request(seq_rows, t, n_tokens);
    const float* end_row = x + (size_t)last * dim;
    float inv_end = inv;
    if (last != t) {                               // the same for the whole block
      __syncthreads();                             // the sums of the request before are read
      inv_end = inverse_rms<G>(end_row, dim, eps, partial[3]);
    }
    const float* kept = inside ? nullptr : rec_copy_before(state, state_stride, dim, slot, positions[t]);
    float* keep = inside ? nullptr : rec_copy_behind(state, state_stride, dim, slot, positions[t] + last - t);
    for (int i = G * threadIdx.x; i < dim; i += G * ST_THREADS) {
      float v[G], p[G], g[G], m[G];
      st_load<G>(row + i, v);
      st_load<G>(gain + i, g);
      st_load<G>(share + i, m);
#pragma unroll
      for (int e = 0; e < G; ++e) v[e] = (v[e] * inv) * g[e];
      if (inside) {
        st_load<G>(row - dim + i, p);
#pragma unroll
        for (int e = 0; e < G; ++e) p[e] = (p[e] * inv_before) * g[e];
      } else {
        st_load<G>(kept + i, p);
        float w[G];
        st_load<G>(end_row + i, w);
#pragma unroll
        for (int e = 0; e < G; ++e) w[e] = (w[e] * inv_end) * g[e];
        st_store<G>(keep + i, w);
      }
#pragma unroll
      for (int e = 0; e < G; ++e) v[e] = fmaf(p[e] - v[e], m[e], v[e]);
      st_store_elem<G>(out + (size_t)t * dim + i, v);
    }
    inv_before = inv;
  }
}

}  // namespace

extern "C" int axk_embed_pairs(const int32_t* tokens, const void* table, int packed, float scale, const void* pairs, int buckets,
                               long mul_prev, long mul_cur, int32_t* state, const int32_t* positions, const int32_t* seq_rows, float* x,
                               int n_tokens, int dim, int vocab, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && dim > 0 && vocab > 0 && buckets > 0 && mul_prev >= 0 && mul_cur >= 0,
              "embed_pairs: bad sizes T=%d dim=%d vocab=%d buckets=%d multipliers %ld %ld", n_tokens, dim, vocab, buckets, mul_prev, mul_cur);
  AXK_REQUIRE(mul_prev < (1L << 31) && mul_cur < (1L << 31), "embed_pairs: multipliers %ld and %ld", mul_prev, mul_cur);
  AXK_REQUIRE(!packed || dim % 32 == 0, "embed_pairs: a packed table has rows of whole blocks of 32, not %d", dim);
  if (n_tokens == 0) return 0;
  embed_pairs_kernel<<<n_tokens, ST_THREADS, 0, (hipStream_t)stream>>>(tokens, (const elem_t*)table, packed, scale, (const elem_t*)pairs,
                                                                       buckets, mul_prev, mul_cur, state, positions, seq_rows, x,
                                                                       n_tokens, dim);
  AXK_LAUNCH_CHECK("embed_pairs");
  return 0;
}

extern "C" int axk_scaled_sum(const float* y0, const float* s0, float norm_eps0, const float* y1, const float* s1, float norm_eps1,
                              float* x, const float* gain, float eps, void* h, const float* share, float* state, long state_stride,
                              const int32_t* positions, const int32_t* seq_rows, int n_tokens, int dim, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && dim > 0 && y0 != nullptr && s0 != nullptr && (y1 == nullptr || s1 != nullptr),
              "scaled_sum: bad sizes T=%d dim=%d, or an output without its scales", n_tokens, dim);
  AXK_REQUIRE(h == nullptr || gain != nullptr, "scaled_sum: a norm without its gain");
  AXK_REQUIRE(share == nullptr || (h != nullptr && state != nullptr && state_stride >= 2L * dim && positions != nullptr && seq_rows != nullptr),
              "scaled_sum: a shift wants the norm and a state of two rows of %d (state rows of %ld)", dim, state_stride);
  if (n_tokens == 0) return 0;
  const bool vec = dim % 4 == 0 && state_stride % 4 == 0 &&
                   (((uintptr_t)y0 | (uintptr_t)s0 | (uintptr_t)y1 | (uintptr_t)s1 | (uintptr_t)x | (uintptr_t)gain | (uintptr_t)h |
                     (uintptr_t)share | (uintptr_t)state) & 15) == 0;
  auto kernel = vec ? scaled_sum_kernel<4> : scaled_sum_kernel<1>;
  kernel<<<n_tokens, ST_THREADS, 0, (hipStream_t)stream>>>(y0, s0, norm_eps0, y1, s1, norm_eps1, x, gain, eps, (elem_t*)h, share, state,
                                                           state_stride, positions, seq_rows, dim);
  AXK_LAUNCH_CHECK("scaled_sum");
  return 0;
}

extern "C" int axk_shifted_norm(const float* x, const float* gain, float eps, const float* share, float* state, long state_stride,
                                const int32_t* positions, const int32_t* seq_rows, void* out, int n_tokens, int dim, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && dim > 0 && gain != nullptr && share != nullptr, "shifted_norm: bad sizes T=%d dim=%d", n_tokens, dim);
  AXK_REQUIRE(state != nullptr && state_stride >= 2L * dim && positions != nullptr && seq_rows != nullptr,
              "shifted_norm: a state row of %ld floats does not hold two rows of %d", state_stride, dim);
  if (n_tokens == 0) return 0;
  const bool vec = dim % 4 == 0 && state_stride % 4 == 0 &&
                   (((uintptr_t)x | (uintptr_t)gain | (uintptr_t)share | (uintptr_t)state | (uintptr_t)out) & 15) == 0;
  const int run = n_tokens >= 4096 ? 4 : 1;       // a row's sum is worked out again by the block behind it: from L2
  auto kernel = vec ? shifted_norm_kernel<4> : shifted_norm_kernel<1>;
  kernel<<<ceil_div(n_tokens, run), ST_THREADS, 0, (hipStream_t)stream>>>(x, gain, eps, share, state, state_stride, positions, seq_rows,
                                                                          (elem_t*)out, n_tokens, dim, run);
  AXK_LAUNCH_CHECK("shifted_norm");
  return 0;
}
