// Shared by the recurrences whose state is a matrix [keys N, values P] per request and head.
//
// A state is kept value by value, [heads][P][N]: the LK lanes that share a value dim hold OWN neighbouring
// rows each, so that a row of the state and a token's key-sized operands are whole vector loads of neighbouring
// lanes.  Rows from N on read as zeros: a state that starts from zeros there stays zero.
//
// A request's state row holds two copies of this and of what else the mixer carries along; the state behind
// position p lives in copy p & 1: a step whose first position is s reads copy (s - 1) & 1 and writes the copy of
// its last position, so a step of one token never writes what it read and gives the same state and output if it
// is run again (a decoding step is run once before it is captured into a graph).  The tokens of a request are
// contiguous in a step and a request is in a step once, so two tokens belong to one request iff their state
// slots (seq_rows) are equal.
#pragma once

#include <math.h>

#include "common.h"

#define REC_THREADS 128

__device__ inline float rec_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ inline float rec_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ inline float rec_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

// The sum over the LK (8 or 16) lanes that share a value dim, in every one of them, by lane permutations of the
// adder: pairs, quads, halves of a row of 16, the row; a fixed order.
template <int LK>
__device__ inline float rec_row_sum(float v) {
#define REC_DPP(val, ctrl) __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, val), ctrl, 0xf, 0xf, false))
  v += REC_DPP(v, 0xb1);                  // quad_perm [1, 0, 3, 2]
  v += REC_DPP(v, 0x4e);                  // quad_perm [2, 3, 0, 1]
  v += REC_DPP(v, 0x141);                 // row_half_mirror
  if (LK == 16) v += REC_DPP(v, 0x140);   // row_mirror
#undef REC_DPP
  return v;
}

// OWN neighbouring floats from row + n0, zeros from N on.  VEC: 16-byte loads (N, n0 and the row's address are
// multiples of 4 floats).
template <int OWN, bool VEC>
__device__ inline void rec_load(float (&dst)[OWN], const float* __restrict__ row, int n0, int N) {
  if (VEC) {
#pragma unroll
    for (int i = 0; i < OWN; i += 4) {
      float4 v = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
      if (n0 + i < N) v = *reinterpret_cast<const float4*>(row + n0 + i);
      dst[i] = v.x; dst[i + 1] = v.y; dst[i + 2] = v.z; dst[i + 3] = v.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < OWN; ++i) dst[i] = n0 + i < N ? row[n0 + i] : 0.0f;
  }
}

template <int OWN, bool VEC>
__device__ inline void rec_store(float* __restrict__ row, const float (&src)[OWN], int n0, int N) {
  if (VEC) {
#pragma unroll
    for (int i = 0; i < OWN; i += 4)
      if (n0 + i < N) *reinterpret_cast<float4*>(row + n0 + i) = make_float4(src[i], src[i + 1], src[i + 2], src[i + 3]);
  } else {
#pragma unroll
    for (int i = 0; i < OWN; ++i)
      if (n0 + i < N) row[n0 + i] = src[i];
  }
}

// The stretch of tokens a block walks: a segment (segs [.][4] = (slot, first token, tokens, whether the request's
// first)), a request's tokens of the step (spans [.][3] = (slot, first token, tokens)), or with neither a token
// that is a request of its own.
struct RecStretch {
  int slot, first, count;
  bool from_state;
};

__device__ inline RecStretch rec_stretch(const int32_t* __restrict__ segs, const int32_t* __restrict__ spans,
                                         const int32_t* __restrict__ seq_rows, int i) {
  if (segs) return RecStretch{segs[4 * i], segs[4 * i + 1], segs[4 * i + 2], segs[4 * i + 3] != 0};
  if (spans) return RecStretch{spans[3 * i], spans[3 * i + 1], spans[3 * i + 2], true};
  return RecStretch{seq_rows[i], i, 1, true};
}

__device__ inline const float* rec_copy_before(const float* state, long state_stride, long copy_elems, int slot, int start) {
  return state + (long)slot * state_stride + (long)((start + 1) & 1) * copy_elems;
}
__device__ inline float* rec_copy_behind(float* state, long state_stride, long copy_elems, int slot, int last) {
  return state + (long)slot * state_stride + (long)(last & 1) * copy_elems;
}

// How many earlier tokens of this step belong to token t's request, up to `most`.
__device__ inline int rec_inside(const int32_t* __restrict__ seq_rows, int t, int most) {
  const int slot = seq_rows[t];
  int inside = 0;
  while (inside < most && t - inside - 1 >= 0 && seq_rows[t - inside - 1] == slot) ++inside;
  return inside;
}

// By the rows of a state: lanes a value dim and rows a lane.
#define REC_BY_ROWS(N, LAUNCH)                \
  {                                           \
    if ((N) <= 32) LAUNCH(8, 4)               \
    else if ((N) <= 64) LAUNCH(16, 4)         \
    else if ((N) <= 128) LAUNCH(16, 8)        \
    else LAUNCH(16, 16)                       \
  }
