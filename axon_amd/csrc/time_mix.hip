// Time mixing with a state matrix a head, decayed per key channel (the time-mix block of RWKV-6-like models):
//
//   token shift   a mix of a token's row and the one before it, h + (h' - h) mu, for each of several uses
//   decay         w = exp(-exp(w0 + W2 tanh(t))), t the low-rank projection of its mix (the kernel of the second product
//                 also makes the delta rule's decays and gates of low rank)
//   per head      o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,  S_t = diag(w_t) S_(t-1) + k_t v_t^T
//
// A copy of the state row (see recurrence.h) holds the heads' states [heads][P][N], then the request's last row
// of the mixer's input (zeros for a new request, which is what the first token's shift reads).
#include "api.h"
#include "recurrence.h"

namespace {

// out[s, t] = h[t] + (h'[t] - h[t]) mu[s], s < n_mix: one read of the rows for all uses, four channels a thread over
// `run` tokens in a row.
__device__ inline void ts_store4(elem_t* dst, const float (&v)[4]) {
#if AXON_BF16
  *reinterpret_cast<uint2*>(dst) = make_uint2(pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]));
#else
  *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
#endif
}

template <int MIXES>        // how many uses, or 0: any number
__global__ void __launch_bounds__(256)
token_shift_kernel(const elem_t* __restrict__ h, const float* __restrict__ mu, int n_mix, const float* __restrict__ state,
                   long state_stride, long copy_elems, long tail_at, const int32_t* __restrict__ positions,
                   const int32_t* __restrict__ seq_rows, elem_t* __restrict__ out, int n_tokens, int width, int run) {
  const int t0 = blockIdx.x * run, t1 = min(t0 + run, n_tokens), c = 4 * (blockIdx.y * 256 + threadIdx.x);
  if (c >= width) return;
  const int valid = min(4, width - c);
  const bool vec = (width & 3) == 0;
  float m[MIXES > 0 ? MIXES : 1][4];
  if (MIXES > 0) {
#pragma unroll
    for (int s = 0; s < MIXES; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i) m[s][i] = i < valid ? mu[(long)s * width + c + i] : 0.0f;
  }
  float prev[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  int slot_before = -1;
  for (int t = t0; t < t1; ++t) {
    const int slot = seq_rows[t];
    if (slot != slot_before) {
      if (t > 0 && seq_rows[t - 1] == slot) {
        load4_guarded(h + (long)(t - 1) * width + c, valid, vec, prev);
      } else {
        const float* kept = rec_copy_before(state, state_stride, copy_elems, slot, positions[t]) + tail_at + c;
#pragma unroll
        for (int i = 0; i < 4; ++i) prev[i] = i < valid ? kept[i] : 0.0f;
      }
      slot_before = slot;
    }
    float cur[4];
    load4_guarded(h + (long)t * width + c, valid, vec, cur);
    const int n = MIXES > 0 ? MIXES : n_mix;
#pragma unroll
    for (int s = 0; s < n; ++s) {
      elem_t* dst = out + ((long)s * n_tokens + t) * width + c;
      float v[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float share = MIXES > 0 ? m[MIXES > 0 ? s : 0][i] : i < valid ? mu[(long)s * width + c + i] : 0.0f;
        v[i] = fmaf(prev[i] - cur[i], share, cur[i]);
      }
      if (vec) ts_store4(dst, v);
      else
        for (int i = 0; i < valid; ++i) dst[i] = from_float(v[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) prev[i] = cur[i];
  }
}

// The second half of low-rank products, out[t, c] = act(sum_k W[c, k] in(low[t, k])), all in 32-bit: tiles of 16 OWN tokens x
// 64 channels, a thread OWN tokens x 4 channels, the rank in pieces of 64 through LDS, a chain in ascending k an output.
// Up to two products of the same tokens share a launch (the first takes the first blocks of a row of the grid).
enum { LR_TIME_MIX_DECAY = 0, LR_DELTA_DECAY = 1, LR_PLAIN = 2 };
struct LowRank {
  const float* low;          // rows of the first half's results
  long low_stride;
  const elem_t* w;           // [channels, rank]
  int channels, rank, kind;
  const void* bias;          // LR_TIME_MIX_DECAY, LR_DELTA_DECAY: [channels]
  int bias_is_f32;
  const void* a_log;         // LR_DELTA_DECAY: one a head of head_dim channels
  int a_log_is_f32, head_dim;
  float* out;                // [T, channels]
};

// in: tanh for LR_TIME_MIX_DECAY, else as it is.
__device__ inline float low_rank_act(const LowRank& r, float v, int c) {
  if (r.kind == LR_PLAIN) return v;
  v += load_vec(r.bias, r.bias_is_f32, c);
  if (r.kind == LR_TIME_MIX_DECAY) return expf(-expf(v));
  return expf(-(expf(load_vec(r.a_log, r.a_log_is_f32, c / r.head_dim)) * rec_softplus(v)));
}

#define TD_CHANNELS 64
#define TD_RANK 64
template <int OWN>
__global__ void __launch_bounds__(256)
low_rank_kernel(LowRank first, LowRank second, int n_tokens) {
  constexpr int TOKENS = 16 * OWN;
  __shared__ __align__(16) float ts[TD_RANK][TOKENS + 4];
  __shared__ __align__(16) float ws[TD_RANK][TD_CHANNELS + 4];
  const int first_blocks = (first.channels + TD_CHANNELS - 1) / TD_CHANNELS;
  const bool is_first = (int)blockIdx.x < first_blocks;
  const LowRank r = is_first ? first : second;
  const int t0 = blockIdx.y * TOKENS, c0 = ((int)blockIdx.x - (is_first ? 0 : first_blocks)) * TD_CHANNELS;
  const int rank = r.rank, channels = r.channels;
  const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
  float acc[OWN][4];
#pragma unroll
  for (int i = 0; i < OWN; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = 0.0f;
  for (int k0 = 0; k0 < rank; k0 += TD_RANK) {
    const int n = min(TD_RANK, rank - k0);
    __syncthreads();
#pragma unroll
    for (int it = 0; it < TOKENS * TD_RANK / 256; ++it) {
      const int i = it * 256 + threadIdx.x, t = i / TD_RANK, k = i % TD_RANK;
      float v = k < n && t0 + t < n_tokens ? r.low[(long)(t0 + t) * r.low_stride + k0 + k] : 0.0f;
      if (r.kind == LR_TIME_MIX_DECAY) v = tanhf(v);
      ts[k][t] = v;
    }
#pragma unroll
    for (int it = 0; it < TD_CHANNELS * TD_RANK / 1024; ++it) {
      const int i = it * 256 + threadIdx.x, c = i / (TD_RANK / 4), k = 4 * (i % (TD_RANK / 4));
      float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
      if (k < n && c0 + c < channels) load4_guarded(r.w + (long)(c0 + c) * rank + k0 + k, n - k, (rank & 3) == 0, v);
#pragma unroll
      for (int j = 0; j < 4; ++j) ws[k + j][c] = v[j];
    }
    __syncthreads();
    const int n_pad = (n + 7) & ~7;
#pragma unroll 8
    for (int k = 0; k < n_pad; ++k) {                // behind the rank: zeros
      const float4 x = *reinterpret_cast<const float4*>(&ws[k][4 * tx]);
#pragma unroll
      for (int i = 0; i < OWN; ++i) {
        const float a = ts[k][OWN * ty + i];
        acc[i][0] = fmaf(a, x.x, acc[i][0]);
        acc[i][1] = fmaf(a, x.y, acc[i][1]);
        acc[i][2] = fmaf(a, x.z, acc[i][2]);
        acc[i][3] = fmaf(a, x.w, acc[i][3]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < OWN; ++i) {
    const int t = t0 + OWN * ty + i;
    if (t >= n_tokens) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = c0 + 4 * tx + j;
      if (c < channels) r.out[(long)t * channels + c] = low_rank_act(r, acc[i][j], c);
    }
  }
}

// The same for up to 16 tokens (a decoding step): 64 channels a block, a lane a channel with 64 of its rank in registers, the
// tokens shared out between the four waves.
#define LF_TOKENS 16
__global__ void __launch_bounds__(256)
low_rank_few_kernel(LowRank first, LowRank second, int n_tokens) {
  __shared__ __align__(16) float ts[LF_TOKENS][TD_RANK];
  const int first_blocks = (first.channels + TD_CHANNELS - 1) / TD_CHANNELS;
  const bool is_first = (int)blockIdx.x < first_blocks;
  const LowRank r = is_first ? first : second;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int c = ((int)blockIdx.x - (is_first ? 0 : first_blocks)) * TD_CHANNELS + lane;
  const elem_t* w = r.w + (long)min(c, r.channels - 1) * r.rank;
  const bool vec = (r.rank & 3) == 0;
  float acc[LF_TOKENS / 4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int k0 = 0; k0 < r.rank; k0 += TD_RANK) {
    const int n = min(TD_RANK, r.rank - k0);
    float x[TD_RANK / 4][4];
#pragma unroll
    for (int i = 0; i < TD_RANK / 4; ++i) load4_guarded(w + k0 + 4 * i, max(0, min(4, n - 4 * i)), vec, x[i]);
    __syncthreads();
    for (int i = threadIdx.x; i < n_tokens * TD_RANK; i += 256) {
      const int t = i / TD_RANK, k = i % TD_RANK;
      float v = k < n ? r.low[(long)t * r.low_stride + k0 + k] : 0.0f;
      if (r.kind == LR_TIME_MIX_DECAY) v = tanhf(v);
      ts[t][k] = v;
    }
    __syncthreads();
#pragma unroll 1
    for (int j = 0; j < LF_TOKENS / 4; ++j) {
      const int t = wave + 4 * j;
      if (t >= n_tokens) break;
      float part[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int i = 0; i < TD_RANK / 4; ++i) {
        const float4 a = *reinterpret_cast<const float4*>(&ts[t][4 * i]);
        part[0] = fmaf(a.x, x[i][0], part[0]);
        part[1] = fmaf(a.y, x[i][1], part[1]);
        part[2] = fmaf(a.z, x[i][2], part[2]);
        part[3] = fmaf(a.w, x[i][3], part[3]);
      }
      const float sum = (part[0] + part[1]) + (part[2] + part[3]);
#pragma unroll
      for (int i = 0; i < LF_TOKENS / 4; ++i)
        if (i == j) acc[i] += sum;
    }
  }
  if (c >= r.channels) return;
#pragma unroll 1
  for (int j = 0; j < LF_TOKENS / 4; ++j) {
    const int t = wave + 4 * j;
    if (t >= n_tokens) break;
    float v = acc[0];
#pragma unroll
    for (int i = 1; i < LF_TOKENS / 4; ++i)
      if (i == j) v = acc[i];
    r.out[(long)t * r.channels + c] = low_rank_act(r, v, c);
  }
}

// The same for many tokens on the 32-bit matrix cores (no tanh on the way in; ranks of whole sixteens): a wave 16 channels x 64
// tokens, rows of W as the first operand, so that a lane holds four neighbouring channels of a token.
typedef __attribute__((ext_vector_type(4))) float lr_f32x4;
__global__ void __launch_bounds__(256)
low_rank_mfma_kernel(LowRank first, LowRank second, int n_tokens) {
  const int first_blocks = (first.channels + TD_CHANNELS - 1) / TD_CHANNELS;
  const bool is_first = (int)blockIdx.x < first_blocks;
  const LowRank r = is_first ? first : second;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, col = lane & 15, g4 = lane >> 4;
  const int c0 = ((int)blockIdx.x - (is_first ? 0 : first_blocks)) * TD_CHANNELS + 16 * wave, t0 = 64 * blockIdx.y;
  if (c0 >= r.channels) return;
  const elem_t* w = r.w + (long)min(c0 + col, r.channels - 1) * r.rank + 4 * g4;
  const float* low[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) low[i] = r.low + (long)min(t0 + 16 * i + col, n_tokens - 1) * r.low_stride + 4 * g4;
  lr_f32x4 acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = lr_f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  for (int k = 0; k < r.rank; k += 32) {
    float a[2][4];
    lr_f32x4 b[2][4];
#pragma unroll
    for (int s = 0; s < 2; ++s)
      if (k + 16 * s < r.rank) {
        load4_guarded(w + k + 16 * s, 4, true, a[s]);
#pragma unroll
        for (int i = 0; i < 4; ++i) b[s][i] = *reinterpret_cast<const lr_f32x4*>(low[i] + k + 16 * s);
      }
#pragma unroll
    for (int s = 0; s < 2; ++s)
      if (k + 16 * s < r.rank)
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[s][j], b[s][i][j], acc[i], 0, 0, 0);
  }
  const int c = c0 + 4 * g4;
  const bool whole = c + 3 < r.channels && (r.channels & 3) == 0;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = t0 + 16 * i + col;
    if (t >= n_tokens) continue;
    float* dst = r.out + (long)t * r.channels + c;
    if (whole) {
      lr_f32x4 v;
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = low_rank_act(r, acc[i][e], c + e);
      *reinterpret_cast<lr_f32x4*>(dst) = v;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < r.channels) dst[e] = low_rank_act(r, acc[i][e], c + e);
    }
  }
}

static bool low_rank_mfma_ok(const LowRank& r) {
  return r.channels == 0 || (r.kind != LR_TIME_MIX_DECAY && r.rank % 16 == 0 && r.low_stride % 4 == 0 && ((uintptr_t)r.low & 15) == 0 &&
                             ((uintptr_t)r.out & 15) == 0);
}

static int launch_low_rank(const LowRank& first, const LowRank& second, int n_tokens, hipStream_t stream, const char* name) {
  const int blocks = ceil_div(first.channels, TD_CHANNELS) + (second.channels > 0 ? ceil_div(second.channels, TD_CHANNELS) : 0);
  if (n_tokens <= LF_TOKENS)
    low_rank_few_kernel<<<blocks, 256, 0, stream>>>(first, second, n_tokens);
  else if (low_rank_mfma_ok(first) && low_rank_mfma_ok(second) && ceil_div(n_tokens, 64) <= 65535)
    low_rank_mfma_kernel<<<dim3(blocks, ceil_div(n_tokens, 64)), 256, 0, stream>>>(first, second, n_tokens);
  else if (n_tokens >= 512)
    low_rank_kernel<4><<<dim3(blocks, ceil_div(n_tokens, 64)), 256, 0, stream>>>(first, second, n_tokens);
  else
    low_rank_kernel<1><<<dim3(blocks, ceil_div(n_tokens, 16)), 256, 0, stream>>>(first, second, n_tokens);
  AXK_LAUNCH_CHECK(name);
  return 0;
}

// The walk.  grid (stretches, heads, blocks of value dims); LK lanes share VP value dims, OWN rows of the state a
// lane.  r, k [T, heads N], v [T, heads P] are columns of rows `stride` apart, w [T, heads N] rows of their own.
// The bonus needs no state: sum_n r_n (S_np + u_n k_n v_p) = sum_n r_n S_np + v_p sum_n r_n u_n k_n.  The operands of
// AHEAD tokens are asked for while those before them are worked on.  In segments (see the launches below) a block
// also leaves rc[t] = r_t times the running product of the segment's earlier w, and the segment's whole product.
template <int OWN, int VP, int AHEAD>
struct WkvOperands {
  float r[AHEAD][OWN], k[AHEAD][OWN], w[AHEAD][OWN], v[AHEAD][VP];
};

#define WKV_VP 2
template <int LK, int OWN, bool VEC>
__global__ void __launch_bounds__(REC_THREADS)
wkv_scan_kernel(const float* __restrict__ rows, long stride, long r_at, long k_at, long v_at, const float* __restrict__ w,
                const float* __restrict__ u, float* __restrict__ state, long state_stride, long copy_elems, long tail_at,
                const int32_t* __restrict__ spans, const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_rows,
                const elem_t* __restrict__ h_in, int width, float* __restrict__ y, int heads, int N, int P,
                const int32_t* __restrict__ segs, float* __restrict__ ends, float* __restrict__ decays, float* __restrict__ rc) {
  constexpr int VP = WKV_VP, AHEAD = OWN >= 16 ? 1 : OWN >= 8 ? 2 : 4;
  const RecStretch s = rec_stretch(segs, spans, seq_rows, blockIdx.x);
  const int h = blockIdx.y, ns = threadIdx.x % LK, n0 = ns * OWN;
  const int p0 = (blockIdx.z * (REC_THREADS / LK) + threadIdx.x / LK) * VP;
  const int start = positions[s.first];
  const float* from = rec_copy_before(state, state_stride, copy_elems, s.slot, start);
  float* to = rec_copy_behind(state, state_stride, copy_elems, s.slot, start + s.count - 1);
  const long s_at = (long)h * N * P;
  float S[VP][OWN], bonus[OWN], D[OWN];
#pragma unroll
  for (int j = 0; j < VP; ++j) {
    if (s.from_state && p0 + j < P) rec_load<OWN, VEC>(S[j], from + s_at + (long)(p0 + j) * N, n0, N);
    else {
#pragma unroll
      for (int i = 0; i < OWN; ++i) S[j][i] = 0.0f;
    }
  }
  rec_load<OWN, VEC>(bonus, u + (long)h * N, n0, N);
#pragma unroll
  for (int i = 0; i < OWN; ++i) D[i] = 1.0f;
  const bool tells = segs != nullptr && blockIdx.z == 0 && threadIdx.x < LK;
  const int last = s.first + s.count;
  const long key = (long)h * N, val = (long)h * P;
  typedef WkvOperands<OWN, VP, AHEAD> Ops;
  auto fetch = [&](Ops& o, int t0) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const int t = min(t0 + a, last - 1);           // behind the last token: the last again, not used
      const float* row = rows + (long)t * stride;
      rec_load<OWN, VEC>(o.r[a], row + r_at + key, n0, N);
      rec_load<OWN, VEC>(o.k[a], row + k_at + key, n0, N);
      rec_load<OWN, VEC>(o.w[a], w + (long)t * heads * N + key, n0, N);
#pragma unroll
      for (int j = 0; j < VP; ++j) o.v[a][j] = row[v_at + val + min(p0 + j, P - 1)];
    }
  };
  auto work = [&](const Ops& o, int t0) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      if (t0 + a >= last) break;
      const int t = t0 + a;
      if (tells) {
        float c[OWN];
#pragma unroll
        for (int i = 0; i < OWN; ++i) { c[i] = o.r[a][i] * D[i]; D[i] *= o.w[a][i]; }
        rec_store<OWN, VEC>(rc + (long)t * heads * N + key, c, n0, N);
      }
      float now = 0.0f;
#pragma unroll
      for (int i = 0; i < OWN; ++i) now = fmaf(o.r[a][i] * bonus[i], o.k[a][i], now);
#pragma unroll
      for (int j = 0; j < VP; ++j) {
        float part = now * o.v[a][j];
#pragma unroll
        for (int i = 0; i < OWN; ++i) {
          part = fmaf(o.r[a][i], S[j][i], part);
          S[j][i] = fmaf(o.w[a][i], S[j][i], o.k[a][i] * o.v[a][j]);
        }
        part = rec_row_sum<LK>(part);
        if (ns == 0 && p0 + j < P) y[(long)t * heads * P + val + p0 + j] = part;
      }
    }
  };
  Ops even, odd;
  fetch(even, s.first);
  for (int t = s.first; t < last; t += 2 * AHEAD) {
    if (t + AHEAD < last) fetch(odd, t + AHEAD);
    work(even, t);
    if (t + AHEAD >= last) break;
    if (t + 2 * AHEAD < last) fetch(even, t + 2 * AHEAD);
    work(odd, t + AHEAD);
  }
  float* into = segs ? ends + ((long)blockIdx.x * heads + h) * N * P : to + s_at;
#pragma unroll
  for (int j = 0; j < VP; ++j)
    if (p0 + j < P) rec_store<OWN, VEC>(into + (long)(p0 + j) * N, S[j], n0, N);
  if (segs) {                   // the request's state is brought up to date by the fold
    if (tells) rec_store<OWN, VEC>(decays + ((long)blockIdx.x * heads + h) * N, D, n0, N);
    return;
  }
  const int n_blocks = gridDim.y * gridDim.z;          // the last row, shared out over the request's blocks
  for (int c = (blockIdx.y * gridDim.z + blockIdx.z) * REC_THREADS + threadIdx.x; c < width; c += n_blocks * REC_THREADS)
    to[tail_at + c] = to_float(h_in[(long)(last - 1) * width + c]);
}

// Long stretches in segments: the walk above runs every segment of a request side by side, the first from the
// request's state, the others from zero.  The fold, an element of the state a thread, goes over a request's segments
// in order: a segment starts from I_1 = E_0, I_(k+1) = diag(D_k) I_k + E_k (left in E_k's place), the last is the
// request's new state.  The carry adds what the state a segment did not start from gives its outputs,
// y_t += I_k^T rc_t; tokens are independent there.  spans5 [n][5] = (slot, first token, tokens, first segment, segments).
#define WKV_CARRY 32        // tokens of a segment a block of the carry takes
__global__ void __launch_bounds__(256)
wkv_fold_kernel(float* __restrict__ ends, const float* __restrict__ decays, const int32_t* __restrict__ spans5,
                float* __restrict__ state, long state_stride, long copy_elems, long tail_at, const int32_t* __restrict__ positions,
                const elem_t* __restrict__ h_in, int width, int heads, int N, int P) {
  const int slot = spans5[5 * blockIdx.x], first = spans5[5 * blockIdx.x + 1], count = spans5[5 * blockIdx.x + 2];
  const int seg0 = spans5[5 * blockIdx.x + 3], n_segs = spans5[5 * blockIdx.x + 4];
  float* to = rec_copy_behind(state, state_stride, copy_elems, slot, positions[first] + count - 1);
  const long i = (long)blockIdx.y * 256 + threadIdx.x, all = (long)heads * N * P;
  if (blockIdx.y == 0)
    for (int c = threadIdx.x; c < width; c += 256) to[tail_at + c] = to_float(h_in[(long)(first + count - 1) * width + c]);
  if (i >= all) return;
  const long d_at = i / ((long)N * P) * N + i % N;
  float I = ends[(long)seg0 * all + i];
  for (int k = 1; k < n_segs; k += 4) {
    float e[4], d[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int seg = seg0 + min(k + j, n_segs - 1);
      e[j] = ends[(long)seg * all + i];
      d[j] = decays[(long)seg * heads * N + d_at];
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (k + j < n_segs) {
        ends[(long)(seg0 + k + j) * all + i] = I;
        I = fmaf(d[j], I, e[j]);
      }
  }
  to[i] = I;
}

template <int LK, int OWN, bool VEC>
__global__ void __launch_bounds__(REC_THREADS)
wkv_carry_kernel(const float* __restrict__ ends, const float* __restrict__ rc, const int32_t* __restrict__ segs,
                 float* __restrict__ y, int heads, int N, int P, int pieces) {
  constexpr int VP = WKV_VP, AHEAD = OWN >= 16 ? 2 : 4;
  const int seg = blockIdx.x / pieces, piece = blockIdx.x % pieces;
  if (segs[4 * seg + 3] != 0) return;                 // a request's first segment started from its state
  const int seg_count = segs[4 * seg + 2];
  if (piece * WKV_CARRY >= seg_count) return;
  const int first = segs[4 * seg + 1] + piece * WKV_CARRY, last = first + min(WKV_CARRY, seg_count - piece * WKV_CARRY);
  const int h = blockIdx.y, ns = threadIdx.x % LK, n0 = ns * OWN;
  const int p0 = (blockIdx.z * (REC_THREADS / LK) + threadIdx.x / LK) * VP;
  float I[VP][OWN];
#pragma unroll
  for (int j = 0; j < VP; ++j) {
    if (p0 + j < P) rec_load<OWN, VEC>(I[j], ends + (((long)seg * heads + h) * P + p0 + j) * N, n0, N);
    else {
#pragma unroll
      for (int i = 0; i < OWN; ++i) I[j][i] = 0.0f;
    }
  }
  for (int t0 = first; t0 < last; t0 += AHEAD) {
    float c[AHEAD][OWN], was[AHEAD][VP];
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const int t = min(t0 + a, last - 1);
      rec_load<OWN, VEC>(c[a], rc + ((long)t * heads + h) * N, n0, N);
#pragma unroll
      for (int j = 0; j < VP; ++j) was[a][j] = y[((long)t * heads + h) * P + min(p0 + j, P - 1)];
    }
#pragma unroll
    for (int a = 0; a < AHEAD; ++a)
#pragma unroll
      for (int j = 0; j < VP; ++j) {
        float part = 0.0f;
#pragma unroll
        for (int i = 0; i < OWN; ++i) part = fmaf(I[j][i], c[a][i], part);
        part = rec_row_sum<LK>(part);
        if (t0 + a < last && ns == 0 && p0 + j < P) y[((long)(t0 + a) * heads + h) * P + p0 + j] = was[a][j] + part;
      }
  }
}

}  // namespace

extern "C" int axk_token_shift(const void* h, const float* mu, int n_mix, const float* state, long state_stride, long copy_elems,
                               long tail_at, const int32_t* positions, const int32_t* seq_rows, void* out, int n_tokens, int width,
                               void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && width > 0 && n_mix > 0, "token_shift: bad sizes T=%d width=%d mixes=%d", n_tokens, width, n_mix);
  AXK_REQUIRE(tail_at >= 0 && copy_elems >= tail_at + width && state_stride >= 2 * copy_elems,
              "token_shift: a state row of %ld floats does not hold two copies of %ld with a row of %d from %ld", state_stride,
              copy_elems, width, tail_at);
  AXK_REQUIRE(((uintptr_t)h & 15) == 0 && ((uintptr_t)out & 15) == 0, "token_shift: rows are not 16-byte aligned");
  if (n_tokens == 0) return 0;
  const int run = n_tokens >= 512 ? 8 : 1;
  auto kernel = n_mix == 5 ? token_shift_kernel<5> : token_shift_kernel<0>;
  kernel<<<dim3(ceil_div(n_tokens, run), ceil_div(width, 1024)), 256, 0, (hipStream_t)stream>>>(
      (const elem_t*)h, mu, n_mix, state, state_stride, copy_elems, tail_at, positions, seq_rows, (elem_t*)out, n_tokens, width, run);
  AXK_LAUNCH_CHECK("token_shift");
  return 0;
}

extern "C" int axk_time_mix_decay(const float* low, const void* w2, const void* w0, int w0_is_f32, float* w, int n_tokens,
                                  int channels, int rank, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && channels > 0 && rank > 0, "time_mix_decay: bad sizes T=%d channels=%d rank=%d", n_tokens, channels, rank);
  AXK_REQUIRE(n_tokens <= 65535 * 16 && ((uintptr_t)w2 & 15) == 0, "time_mix_decay: %d tokens in one step, or w2 is not aligned", n_tokens);
  if (n_tokens == 0) return 0;
  const LowRank job = {low, rank, (const elem_t*)w2, channels, rank, LR_TIME_MIX_DECAY, w0, w0_is_f32, nullptr, 0, 1, w};
  LowRank none = job;
  none.channels = 0;
  return launch_low_rank(job, none, n_tokens, (hipStream_t)stream, "time_mix_decay");
}

extern "C" int axk_delta_low_rank(const float* rows, long stride, int decay_at, int decay_rank, const void* w_decay, const void* dt_bias,
                                  int dt_bias_is_f32, const void* a_log, int a_log_is_f32, int head_dim, float* decay,
                                  int decay_channels, int gate_at, int gate_rank, const void* w_gate, float* gate, int gate_channels,
                                  int n_tokens, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && decay_channels >= 0 && gate_channels >= 0 && decay_channels + gate_channels > 0 &&
              n_tokens <= 65535 * 16, "delta_low_rank: bad sizes T=%d channels=%d, %d", n_tokens, decay_channels, gate_channels);
  AXK_REQUIRE(decay_channels == 0 || (decay_rank > 0 && decay_at >= 0 && decay_at + (long)decay_rank <= stride && head_dim > 0 &&
                                      ((uintptr_t)w_decay & 15) == 0),
              "delta_low_rank: decays of rank %d from column %d of %ld, heads of %d", decay_rank, decay_at, stride, head_dim);
  AXK_REQUIRE(gate_channels == 0 || (gate_rank > 0 && gate_at >= 0 && gate_at + (long)gate_rank <= stride && ((uintptr_t)w_gate & 15) == 0),
              "delta_low_rank: gates of rank %d from column %d of %ld", gate_rank, gate_at, stride);
  if (n_tokens == 0) return 0;
  const LowRank d = {rows + decay_at, stride, (const elem_t*)w_decay, decay_channels, decay_rank, LR_DELTA_DECAY, dt_bias, dt_bias_is_f32,
                     a_log, a_log_is_f32, head_dim, decay};
  const LowRank g = {rows + gate_at, stride, (const elem_t*)w_gate, gate_channels, gate_rank, LR_PLAIN, nullptr, 0, nullptr, 0, 1, gate};
  return launch_low_rank(d, g, n_tokens, (hipStream_t)stream, "delta_low_rank");
}

extern "C" int axk_wkv_scan(const float* rows, long stride, long r_at, long k_at, long v_at, const float* w, const float* u,
                            float* state, long state_stride, long copy_elems, long tail_at, const int32_t* spans, int n_spans,
                            const int32_t* positions, const int32_t* seq_rows, const void* h_in, int width, float* y, int heads,
                            int N, int P, const int32_t* segs, int n_segs, int longest_seg, const int32_t* spans5, float* ends,
                            float* decays, float* rc, void* stream) {
  AXK_REQUIRE(n_spans >= 0 && heads > 0 && N > 0 && N <= 256 && P > 0 && width > 0,
              "wkv_scan: bad sizes spans=%d heads=%d keys=%d (at most 256) values=%d", n_spans, heads, N, P);
  AXK_REQUIRE(r_at >= 0 && k_at >= 0 && v_at >= 0 && r_at + (long)heads * N <= stride && k_at + (long)heads * N <= stride &&
              v_at + (long)heads * P <= stride, "wkv_scan: the parts do not fit rows of %ld", stride);
  AXK_REQUIRE(tail_at >= (long)heads * N * P && copy_elems >= tail_at + width && state_stride >= 2 * copy_elems,
              "wkv_scan: a state row of %ld floats does not hold two copies of %ld (%d x %d x %d, then %d from %ld)", state_stride,
              copy_elems, heads, N, P, width, tail_at);
  AXK_REQUIRE((spans != nullptr || seq_rows != nullptr) && positions != nullptr, "wkv_scan: neither spans nor slots, or no positions");
  AXK_REQUIRE(segs == nullptr || (n_segs >= n_spans && longest_seg > 0 && spans5 != nullptr && ends != nullptr && decays != nullptr &&
                                  rc != nullptr && spans != nullptr),
              "wkv_scan: %d segments of %d requests come with the requests' list and their workspaces", n_segs, n_spans);
  if (n_spans == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = N % 4 == 0 && stride % 4 == 0 && r_at % 4 == 0 && k_at % 4 == 0 && copy_elems % 4 == 0 && state_stride % 4 == 0 &&
                   ((uintptr_t)rows & 15) == 0 && ((uintptr_t)w & 15) == 0 && ((uintptr_t)u & 15) == 0 && ((uintptr_t)state & 15) == 0 &&
                   ((uintptr_t)ends & 15) == 0 && ((uintptr_t)decays & 15) == 0 && ((uintptr_t)rc & 15) == 0;
  const int pieces = segs ? ceil_div(longest_seg, WKV_CARRY) : 1;
#define WKV_ARGS rows, stride, r_at, k_at, v_at, w, u, state, state_stride, copy_elems, tail_at, spans, positions, seq_rows, \
                 (const elem_t*)h_in, width, y, heads, N, P, segs, ends, decays, rc
#define WKV_LAUNCH(LK, OWN)                                                                                             \
  {                                                                                                                     \
    const int z = ceil_div(P, REC_THREADS / LK * WKV_VP);                                                               \
    const dim3 grid(segs ? n_segs : n_spans, heads, z), carry((unsigned)((long)(segs ? n_segs : 1) * pieces), heads, z); \
    if (vec) wkv_scan_kernel<LK, OWN, true><<<grid, REC_THREADS, 0, s>>>(WKV_ARGS);                                     \
    else wkv_scan_kernel<LK, OWN, false><<<grid, REC_THREADS, 0, s>>>(WKV_ARGS);                                        \
    if (segs) {                                                                                                         \
      const dim3 fold(n_spans, (unsigned)(((long)heads * N * P + 255) / 256));                                          \
      wkv_fold_kernel<<<fold, 256, 0, s>>>(ends, decays, spans5, state, state_stride, copy_elems, tail_at, positions,   \
                                           (const elem_t*)h_in, width, heads, N, P);                                    \
      if (vec) wkv_carry_kernel<LK, OWN, true><<<carry, REC_THREADS, 0, s>>>(ends, rc, segs, y, heads, N, P, pieces);   \
      else wkv_carry_kernel<LK, OWN, false><<<carry, REC_THREADS, 0, s>>>(ends, rc, segs, y, heads, N, P, pieces);      \
    }                                                                                                                   \
  }
  REC_BY_ROWS(N, WKV_LAUNCH)
#undef WKV_LAUNCH
#undef WKV_ARGS
  AXK_LAUNCH_CHECK("wkv_scan");
  return 0;
}
