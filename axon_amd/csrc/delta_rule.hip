// The gated delta rule (the linear attention of Gated-DeltaNet-like models): per request and head a state matrix
// S [N, P] that each token decays, corrects along its key and reads,
//
//   S <- g_t S,  u = beta_t (v_t - S^T k_t),  S <- S + k_t u^T,  o_t = S^T q_t,
//
// behind short causal convolutions with silu over the channels [q | k | v], queries and keys of length 1 a head.
// Head a reads query and key head a / (heads / kv_heads).  Everything here is 32-bit in both builds but the
// convolutions' weights as stored.
//
// A copy of the state row (see recurrence.h) holds the heads' states [heads][P][N], then [taps - 1][channels] of the
// convolutions' last inputs, oldest first (zeros for a new request, which is what they read before the first token).
#include "api.h"
#include "recurrence.h"

namespace {

// A wave a unit of a token: a query or key head (convolution, silu, length 1; queries also times N^(-1/2)), a value
// head (convolution, silu), or the token's step sizes, terms[t, a] = (g, beta) with
// g = exp(-exp(A_log_a) softplus(decay_in_a + dt_bias_a)), beta = sigmoid(beta_in_a).  in [T, in_stride]: the
// projections' rows, [q: kv_heads N | k: kv_heads N | v: heads P] first.
// Without a_log (a decay a key channel, which comes from elsewhere) g is 1.
__device__ inline float delta_decay(const float* __restrict__ row, int decay_at, const void* __restrict__ a_log, int a_log_is_f32,
                                    const void* __restrict__ dt_bias, int dt_bias_is_f32, int a) {
  if (a_log == nullptr) return 1.0f;
  const float step = rec_softplus(row[decay_at + a] + load_vec(dt_bias, dt_bias_is_f32, a));
  return expf(-(expf(load_vec(a_log, a_log_is_f32, a)) * step));
}

#define DP_KEPT 4        // channels of a query or key head a lane holds: N up to 256
__global__ void __launch_bounds__(256)
delta_prepare_kernel(const float* __restrict__ in, long in_stride, const elem_t* __restrict__ w, int taps,
                     const float* __restrict__ state, long state_stride, long copy_elems, long tail_at,
                     const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_rows, int beta_at, int decay_at,
                     const void* __restrict__ a_log, int a_log_is_f32, const void* __restrict__ dt_bias, int dt_bias_is_f32,
                     float* __restrict__ u, float* __restrict__ terms, int heads, int kv_heads, int N, int P, float q_scale) {
  const int t = blockIdx.x, unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const float* row = in + (long)t * in_stride;
  if (unit > 2 * kv_heads + heads) return;
  if (unit == 2 * kv_heads + heads) {
    for (int a = lane; a < heads; a += 64) {
      terms[((long)t * heads + a) * 2] = delta_decay(row, decay_at, a_log, a_log_is_f32, dt_bias, dt_bias_is_f32, a);
      terms[((long)t * heads + a) * 2 + 1] = rec_sigmoid(row[beta_at + a]);
    }
    return;
  }
  const int channels = 2 * kv_heads * N + heads * P;
  const bool is_v = unit >= 2 * kv_heads;
  const int c0 = is_v ? 2 * kv_heads * N + (unit - 2 * kv_heads) * P : unit * N, size = is_v ? P : N;
  const int inside = rec_inside(seq_rows, t, taps - 1);
  const float* kept = rec_copy_before(state, state_stride, copy_elems, seq_rows[t], positions[t] - inside) + tail_at;
  auto conv = [&](int c) {
    float acc = 0.0f;
    for (int k = 0; k < taps; ++k) {
      const int back = taps - 1 - k;            // the input `back` tokens before this one
      const float v = back <= inside ? row[c - (long)back * in_stride]
                                     : kept[(long)(taps - 1 - (back - inside)) * channels + c];
      acc = fmaf(to_float(w[(long)c * taps + k]), v, acc);
    }
    return rec_silu(acc);
  };
  float* dst = u + (long)t * channels;
  if (is_v) {
    for (int i = lane; i < size; i += 64) dst[c0 + i] = conv(c0 + i);
    return;
  }
  float v[DP_KEPT], ss = 0.0f;
#pragma unroll
  for (int j = 0; j < DP_KEPT; ++j) {
    v[j] = lane + 64 * j < size ? conv(c0 + lane + 64 * j) : 0.0f;
    ss = fmaf(v[j], v[j], ss);
  }
  const float inv = (1.0f / sqrtf(wave_sum(ss) + 1e-6f)) * (unit < kv_heads ? q_scale : 1.0f);
#pragma unroll
  for (int j = 0; j < DP_KEPT; ++j)
    if (lane + 64 * j < size) dst[c0 + lane + 64 * j] = v[j] * inv;
}

// The convolutions' last taps - 1 inputs: of (what was kept, this step's inputs) the last taps - 1; place i takes what
// lies `count` places later (where both copies are one: read before it is written, ascending).  The channels are shared
// out over a request's threads, this being the one numbered `me` of `all`.
__device__ inline void keep_conv_inputs(const float* __restrict__ kept_from, float* kept, const float* __restrict__ conv_in,
                                        long conv_in_stride, int first, int count, int channels, int taps, int me, int all) {
  for (int c = me; c < channels; c += all)
    for (int i = 0; i < taps - 1; ++i) {
      const int at = i + count;
      kept[(long)i * channels + c] = at < taps - 1 ? kept_from[(long)at * channels + c]
                                                   : conv_in[(long)(first + at - (taps - 1)) * conv_in_stride + c];
    }
}

// The walk.  grid (requests of the step, heads, blocks of value dims); LK lanes share a value dim, OWN rows of the
// state a lane.  With a = S^T k and b = S^T q of the state as the token finds it, u = beta (v - g a) and the read-out
// behind the token's write is o = g b + (k . q) u: both sums leave for the lanes' permutations together.  The operands
// of AHEAD tokens are asked for while those before them are worked on.  CHANNEL: a decay a head and key channel, from
// decay [T, heads N] (the state's rows are then decayed before the sums, and g is 1).
template <int OWN, int AHEAD, bool CHANNEL>
struct DeltaOperands {
  float q[AHEAD][OWN], k[AHEAD][OWN], v[AHEAD], g[AHEAD], beta[AHEAD], w[CHANNEL ? AHEAD : 1][OWN];
};

template <int LK, int OWN, bool VEC, bool CHANNEL>
__global__ void __launch_bounds__(REC_THREADS)
delta_scan_kernel(const float* __restrict__ u, const float* __restrict__ terms, const float* __restrict__ decay, float* __restrict__ state, long state_stride,
                  long copy_elems, long tail_at, const int32_t* __restrict__ spans, const int32_t* __restrict__ positions,
                  const int32_t* __restrict__ seq_rows, const float* __restrict__ conv_in, long conv_in_stride,
                  float* __restrict__ y, int heads, int kv_heads, int N, int P, int taps) {
  constexpr int AHEAD = OWN >= 16 ? 2 : 4;
  const RecStretch s = rec_stretch(nullptr, spans, seq_rows, blockIdx.x);
  const int h = blockIdx.y, kh = h / (heads / kv_heads), ns = threadIdx.x % LK, n0 = ns * OWN;
  const int p = blockIdx.z * (REC_THREADS / LK) + threadIdx.x / LK;
  const bool has_p = p < P;
  const int start = positions[s.first];
  const float* from = rec_copy_before(state, state_stride, copy_elems, s.slot, start);
  float* to = rec_copy_behind(state, state_stride, copy_elems, s.slot, start + s.count - 1);
  const long s_at = (long)h * N * P + (long)p * N;
  float S[OWN];
  if (has_p) rec_load<OWN, VEC>(S, from + s_at, n0, N);
  else {
#pragma unroll
    for (int i = 0; i < OWN; ++i) S[i] = 0.0f;
  }
  const int channels = 2 * kv_heads * N + heads * P, last = s.first + s.count;
  const long q_col = (long)kh * N, k_col = (long)(kv_heads + kh) * N, v_col = 2L * kv_heads * N + (long)h * P + (has_p ? p : 0);
  typedef DeltaOperands<OWN, AHEAD, CHANNEL> Ops;
  auto fetch = [&](Ops& o, int t0) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const int t = min(t0 + a, last - 1);             // behind the last token: the last again, not used
      const float* row = u + (long)t * channels;
      rec_load<OWN, VEC>(o.q[a], row + q_col, n0, N);
      rec_load<OWN, VEC>(o.k[a], row + k_col, n0, N);
      if (CHANNEL) rec_load<OWN, VEC>(o.w[CHANNEL ? a : 0], decay + ((long)t * heads + h) * N, n0, N);
      o.v[a] = row[v_col];
      o.g[a] = terms[((long)t * heads + h) * 2];
      o.beta[a] = terms[((long)t * heads + h) * 2 + 1];
    }
  };
  auto work = [&](const Ops& o, int t0) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      if (t0 + a >= last) break;
      float sk = 0.0f, sq = 0.0f, kq = 0.0f;
      const float g = CHANNEL ? 1.0f : o.g[a];
#pragma unroll
      for (int i = 0; i < OWN; ++i) {
        if (CHANNEL) S[i] *= o.w[CHANNEL ? a : 0][i];
        sk = fmaf(S[i], o.k[a][i], sk);
        sq = fmaf(S[i], o.q[a][i], sq);
        kq = fmaf(o.k[a][i], o.q[a][i], kq);
      }
      sk = rec_row_sum<LK>(sk);
      sq = rec_row_sum<LK>(sq);
      kq = rec_row_sum<LK>(kq);
      const float c = o.beta[a] * (o.v[a] - g * sk);
#pragma unroll
      for (int i = 0; i < OWN; ++i) S[i] = fmaf(o.k[a][i], c, g * S[i]);
      if (ns == 0 && has_p) y[((long)(t0 + a) * heads + h) * P + p] = fmaf(kq, c, g * sq);
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
  if (has_p) rec_store<OWN, VEC>(to + s_at, S, n0, N);
  keep_conv_inputs(from + tail_at, to + tail_at, conv_in, conv_in_stride, s.first, s.count, channels, taps,
                   (blockIdx.y * gridDim.z + blockIdx.z) * REC_THREADS + threadIdx.x, gridDim.y * gridDim.z * REC_THREADS);
}

// Long stretches in chunks of 64 tokens, on the 32-bit matrix cores.  Inside a chunk that finds the state S, with
// b_i the product of the chunk's g up to token i, D_ij = g_(j+1) ... g_i and A_ij = beta_i D_ij (k_i . k_j) for j < i,
// the tokens' corrections solve a unit lower triangular system that the state enters linearly:
//   (I + A) U = diag(beta) V - diag(beta b) K S,     U = U' - W S,
//   O = diag(b) Q S + M U,  M_ij = D_ij (q_i . k_j) for j <= i,     S <- b_last S + (diag(D_last) K)^T U.
// The first kernel makes U', W, M and the scaled transposed keys of every (chunk, head) side by side: the products
// k_i . k_j and q_i . k_j by MFMA, the products of decays one multiplication after the other (never a quotient, so a
// decay of 0 is nothing special), the two right-hand sides by forward substitution, a column a thread with its 64 rows
// in registers.  The second walks a request's chunks per (head, sixteen value dims).  The sums of a token are those of
// the walk token by token in another order.
// Of a (chunk, head), item = chunk heads + head: U' [64][P] and b [64] row by row; W [64][N], M [64][64] (its upper tiles
// are not written) and kt [N][64], and of a (chunk, query head) Q [64][N], as the walk's operands, tile of sixteen rows
// by tile, sixteen columns by sixteen, in the order of a wave's lanes (dc_at): a load of four floats a lane then reads
// 1 KB side by side.  Rows beyond the chunk's tokens have g 1 and beta 0: they change nothing.
#define DC 64
typedef __attribute__((ext_vector_type(4))) float dc_f32x4;
__device__ inline dc_f32x4 dc_load(const float* p) { return *reinterpret_cast<const dc_f32x4*>(p); }
// where a matrix of 16 cols16 columns keeps (row, col): lane l = row % 16 + 16 (col % 16 / 4) of block (row / 16, col / 16)
__device__ inline long dc_at(int row, int col, int cols16) {
  return ((long)(row / 16 * cols16 + col / 16) * 64 + row % 16 + 16 * (col % 16 / 4)) * 4 + col % 4;
}
// sixteen k of a product are four chained instructions: lane l holds rows l % 16 at k = 4 (l / 16) .. + 3 of either
// operand, instruction j takes their j-th.  Independent chains run interleaved, so that none waits for itself.
#define DC_MFMA(acc, a, b, j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32((a)[j], (b)[j], acc, 0, 0, 0)

template <int NT>
__global__ void __launch_bounds__(256)
delta_chunk_terms_kernel(const float* __restrict__ u, const float* __restrict__ terms, const int32_t* __restrict__ chunks, int heads,
                         int kv_heads, int P, float* __restrict__ up, float* __restrict__ w, float* __restrict__ kt,
                         float* __restrict__ m, float* __restrict__ q, float* __restrict__ b) {
  constexpr int N = 16 * NT, ROW = DC + 4;
  __shared__ float D[DC][DC + 1];
  __shared__ __align__(16) float A[DC][ROW];
  __shared__ float gs[DC], betas[DC], bs[DC];
  const int h = blockIdx.x, kh = h / (heads / kv_heads), first = chunks[2 * blockIdx.y], count = chunks[2 * blockIdx.y + 1];
  const long item = (long)blockIdx.y * heads + h;
  const int channels = 2 * kv_heads * N + heads * P;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 15, g4 = lane >> 4;
  if (tid < DC) {
    gs[tid] = tid < count ? terms[((long)(first + tid) * heads + h) * 2] : 1.0f;
    betas[tid] = tid < count ? terms[((long)(first + tid) * heads + h) * 2 + 1] : 0.0f;
  }
  __syncthreads();
  if (tid < DC) {
    float d = 1.0f;
    D[tid][tid] = 1.0f;
    for (int i = tid + 1; i < DC; ++i) { d *= gs[i]; D[i][tid] = d; }
  } else if (tid == DC) {
    float d = 1.0f;
    for (int i = 0; i < DC; ++i) { d *= gs[i]; bs[i] = d; b[item * DC + i] = d; }
  }
  const float* keys = u + (long)(kv_heads + kh) * N;
  const float* mine = u + (long)(first + min(16 * wave + r, count - 1)) * channels + (long)kh * N + 4 * g4;
  dc_f32x4 qf[NT], kf[NT];
#pragma unroll
  for (int c = 0; c < NT; ++c) { qf[c] = dc_load(mine + 16 * c); kf[c] = dc_load(mine + (long)kv_heads * N + 16 * c); }
  if (h % (heads / kv_heads) == 0) {
    float* dst = q + ((long)blockIdx.y * kv_heads + kh) * DC * N;
#pragma unroll
    for (int c = 0; c < NT; ++c) *reinterpret_cast<dc_f32x4*>(dst + ((wave * NT + c) * 64 + lane) * 4) = qf[c];
  }
  __syncthreads();
  for (int jt = 0; jt <= wave; ++jt) {
    const float* other = keys + (long)(first + min(16 * jt + r, count - 1)) * channels + 4 * g4;
    dc_f32x4 kk = {0.0f, 0.0f, 0.0f, 0.0f}, qk = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int c = 0; c < NT; ++c) {
      const dc_f32x4 o = dc_load(other + 16 * c);
#pragma unroll
      for (int j = 0; j < 4; ++j) { DC_MFMA(kk, kf[c], o, j); DC_MFMA(qk, qf[c], o, j); }
    }
    const int j = 16 * jt + r;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * wave + 4 * g4 + e;
      A[i][j] = j < i ? (betas[i] * D[i][j]) * kk[e] : 0.0f;
      m[item * DC * DC + dc_at(i, j, DC / 16)] = j <= i ? D[i][j] * qk[e] : 0.0f;
    }
  }
  __syncthreads();
  const int cols = P + N;
  for (int col = tid; col < cols; col += 256) {
    float X[DC];
    const bool is_v = col < P;
    const float* src = u + (is_v ? 2L * kv_heads * N + (long)h * P + col : (long)(kv_heads + kh) * N + col - P);
#pragma unroll
    for (int i = 0; i < DC; ++i) X[i] = src[(long)(first + min(i, count - 1)) * channels];
    if (!is_v) {
      float* dst = kt + item * N * DC;
#pragma unroll
      for (int i = 0; i < DC; i += 4)
        *reinterpret_cast<dc_f32x4*>(dst + dc_at(col - P, i, DC / 16)) = dc_f32x4{X[i] * D[DC - 1][i], X[i + 1] * D[DC - 1][i + 1], X[i + 2] * D[DC - 1][i + 2],
                                                         X[i + 3] * D[DC - 1][i + 3]};
    }
#pragma unroll
    for (int i = 0; i < DC; ++i) X[i] *= is_v ? betas[i] : betas[i] * bs[i];
#pragma unroll
    for (int i = 1; i < DC; ++i) {
      float x = X[i];
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const dc_f32x4 a = dc_load(&A[i][j]);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j + e < i) x = fmaf(-a[e], X[j + e], x);
      }
      X[i] = x;
      __builtin_amdgcn_sched_barrier(0);       // a row of A at a time in registers
    }
    if (is_v) {
      float* dst = up + item * DC * P + col;
#pragma unroll
      for (int i = 0; i < DC; ++i) dst[(long)i * P] = X[i];
    } else {
      float* dst = w + item * DC * N;
#pragma unroll
      for (int i = 0; i < DC; ++i) dst[dc_at(i, col - P, NT)] = X[i];
    }
  }
}

// The same with a decay a key channel: D_ij and b_i are vectors over the channels, (k_i . k_j) and (q_i . k_j) become sums of
// k_in D_ijn k_jn.  Such a sum is a product of two rows once D_ij is cut at a place x between the tokens: (the decays of
// x .. i) times (those of j + 1 .. x - 1), both products of factors up to 1, so nothing overflows and nothing is divided.
// Two tokens are cut where their numbers first differ: with s the highest bit in which i and j differ, x is the start of i's
// run of s tokens, and a token's factor at level s is the product from its run's start to itself where bit s is set in its
// number (`pre`), else from behind itself to its run's end (`suf`).  So each level is one scaling of the rows and one
// product, of which the pairs that belong to the level are taken: levels 1 to 8 inside a wave's sixteen tokens, 16 and 32
// between waves.  Level by level pre and suf double their reach by the neighbouring run's whole product.
// Of a (chunk, head) q holds diag(b_i) q_i and b the last token's b [N].
// Of sixteen lanes in runs of s: the value that the neighbouring run's last lane holds, by lane permutations.
__device__ inline float dc_neighbour_run(float v, int s, bool second_quad) {
#define DC_DPP(val, ctrl) __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, val), ctrl, 0xf, 0xf, false))
  if (s == 1) return DC_DPP(v, 0xb1);                        // quad_perm [1, 0, 3, 2]
  if (s == 2) return DC_DPP(v, 0x5f);                        // quad_perm [3, 3, 1, 1]
  const float last = DC_DPP(v, 0xff);                        // of a lane's own four: quad_perm [3, 3, 3, 3]
  const float other = DC_DPP(last, 0x141);                   // of the other four of its eight: row_half_mirror
  if (s == 4) return other;
  return DC_DPP(second_quad ? last : other, 0x140);          // of the other eight: row_mirror
#undef DC_DPP
}

template <int NT>
__global__ void __launch_bounds__(256, 2)        // two waves a SIMD: 256 registers each
delta_chunk_channel_terms_kernel(const float* __restrict__ u, const float* __restrict__ terms, const float* __restrict__ decay,
                                 const int32_t* __restrict__ chunks, int heads, int kv_heads, int P, float* __restrict__ up,
                                 float* __restrict__ w, float* __restrict__ kt, float* __restrict__ m, float* __restrict__ q,
                                 float* __restrict__ b) {
  constexpr int N = 16 * NT, ROW = DC + 4, KROW = N + 4;
  __shared__ __align__(16) float Kl[DC][KROW];        // rows 0 .. 31: level 16 of waves 0 and 2; 32 .. 63: level 32 of waves 0 and 1
  __shared__ __align__(16) float A[DC][ROW];
  __shared__ __align__(16) float tot[4][N];
  __shared__ float betas[DC];
  const int h = blockIdx.x, kh = h / (heads / kv_heads), first = chunks[2 * blockIdx.y], count = chunks[2 * blockIdx.y + 1];
  const long item = (long)blockIdx.y * heads + h;
  const int channels = 2 * kv_heads * N + heads * P;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 15, g4 = lane >> 4, row = 16 * wave + r;
  if (tid < DC) betas[tid] = tid < count ? terms[((long)(first + tid) * heads + h) * 2 + 1] : 0.0f;
  const long t = first + min(row, count - 1);
  const float* mine = u + t * channels + (long)kh * N + 4 * g4;
  const float* mine_g = decay + (t * heads + h) * N + 4 * g4;
  dc_f32x4 qf[NT], kf[NT], pre[NT], suf[NT];
  float own = 0.0f;                                   // q_i . k_i, nothing decayed
#pragma unroll
  for (int c = 0; c < NT; ++c) {
    qf[c] = dc_load(mine + 16 * c);
    kf[c] = dc_load(mine + (long)kv_heads * N + 16 * c);
    pre[c] = row < count ? dc_load(mine_g + 16 * c) : dc_f32x4{1.0f, 1.0f, 1.0f, 1.0f};
    suf[c] = dc_f32x4{1.0f, 1.0f, 1.0f, 1.0f};
#pragma unroll
    for (int j = 0; j < 4; ++j) own = fmaf(qf[c][j], kf[c][j], own);
  }
  own += __shfl_xor(own, 16, 64);
  own += __shfl_xor(own, 32, 64);
  dc_f32x4 kk = {0.0f, 0.0f, 0.0f, 0.0f}, qk = kk;
#pragma unroll
  for (int s = 1; s < 16; s <<= 1) {
    const bool high = (r & s) != 0;
    dc_f32x4 ks = {0.0f, 0.0f, 0.0f, 0.0f}, qs = ks;
#pragma unroll
    for (int c = 0; c < NT; ++c) {
      const dc_f32x4 f = high ? pre[c] : suf[c], kd = kf[c] * f, qd = qf[c] * f;
#pragma unroll
      for (int j = 0; j < 4; ++j) { DC_MFMA(ks, kd, kd, j); DC_MFMA(qs, qd, kd, j); }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 4 * g4 + e, x = i ^ r;            // row i, column r
      if ((i & s) != 0 && (x & s) != 0 && x < 2 * s) { kk[e] = ks[e]; qk[e] = qs[e]; }
    }
#pragma unroll
    for (int c = 0; c < NT; ++c)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float whole = dc_neighbour_run(pre[c][j], s, (r & 4) != 0);
        pre[c][j] *= high ? whole : 1.0f;
        suf[c][j] *= high ? 1.0f : whole;
      }
  }
  // pre and suf now reach over the wave's tokens
  if (r == 15) {
#pragma unroll
    for (int c = 0; c < NT; ++c) *reinterpret_cast<dc_f32x4*>(&tot[wave][16 * c + 4 * g4]) = pre[c];
  }
  if ((wave & 1) == 0) {
#pragma unroll
    for (int c = 0; c < NT; ++c) *reinterpret_cast<dc_f32x4*>(&Kl[8 * wave + r][16 * c + 4 * g4]) = kf[c] * suf[c];
  }
  __syncthreads();
  auto tile = [&](int jt, dc_f32x4 kd, dc_f32x4 qd) {          // rows of this wave, columns 16 jt ..
    const int j = 16 * jt + r;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * wave + 4 * g4 + e;
      A[i][j] = j < i ? betas[i] * kd[e] : 0.0f;
      m[item * DC * DC + dc_at(i, j, DC / 16)] = j < i ? qd[e] : j == i ? own : 0.0f;
    }
  };
  auto product = [&](int jt, const float (*rows)[KROW]) {      // rows: the columns' tokens, scaled; pre: this wave's factors
    dc_f32x4 ks = {0.0f, 0.0f, 0.0f, 0.0f}, qs = ks;
#pragma unroll
    for (int c = 0; c < NT; ++c) {
      const dc_f32x4 o = dc_load(&rows[r][16 * c + 4 * g4]), kd = kf[c] * pre[c], qd = qf[c] * pre[c];
#pragma unroll
      for (int j = 0; j < 4; ++j) { DC_MFMA(ks, kd, o, j); DC_MFMA(qs, qd, o, j); }
    }
    tile(jt, ks, qs);
  };
  tile(wave, kk, qk);
  if (wave & 1) product(wave - 1, &Kl[8 * (wave - 1)]);
#pragma unroll
  for (int c = 0; c < NT; ++c) {
    const dc_f32x4 whole = dc_load(&tot[wave ^ 1][16 * c + 4 * g4]);
    if (wave & 1) pre[c] *= whole; else suf[c] *= whole;
    if (wave < 2) *reinterpret_cast<dc_f32x4*>(&Kl[32 + row][16 * c + 4 * g4]) = kf[c] * suf[c];
  }
  __syncthreads();
  if (wave & 2) {
    product(0, &Kl[32]);
    product(1, &Kl[48]);
  }
#pragma unroll
  for (int c = 0; c < NT; ++c) {
    const int other = wave & 2 ? 0 : 2;
    const dc_f32x4 whole = dc_load(&tot[other][16 * c + 4 * g4]) * dc_load(&tot[other + 1][16 * c + 4 * g4]);
    if (wave & 2) pre[c] *= whole; else suf[c] *= whole;
  }
  __syncthreads();                                   // the scaled rows have been read
  // now over the whole chunk: q and the last decays as the walk wants them, the keys transposed, and the right-hand side
#pragma unroll
  for (int c = 0; c < NT; ++c) {
    *reinterpret_cast<dc_f32x4*>(q + item * DC * N + ((wave * NT + c) * 64 + lane) * 4) = qf[c] * pre[c];
    *reinterpret_cast<dc_f32x4*>(&Kl[row][16 * c + 4 * g4]) = (kf[c] * pre[c]) * betas[row];
    if (row == DC - 1) *reinterpret_cast<dc_f32x4*>(b + item * N + 16 * c + 4 * g4) = pre[c];
    const dc_f32x4 kd = kf[c] * suf[c];
#pragma unroll
    for (int j = 0; j < 4; ++j) kt[item * N * DC + dc_at(16 * c + 4 * g4 + j, row, DC / 16)] = kd[j];
  }
  __syncthreads();
  const int cols = P + N;
  for (int col = tid; col < cols; col += 256) {
    float X[DC];
    const bool is_v = col < P;
    const float* src = u + 2L * kv_heads * N + (long)h * P + (is_v ? col : 0);
#pragma unroll
    for (int i = 0; i < DC; ++i) X[i] = is_v ? src[(long)(first + min(i, count - 1)) * channels] * betas[i] : Kl[i][is_v ? 0 : col - P];
#pragma unroll
    for (int i = 1; i < DC; ++i) {
      float x = X[i];
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const dc_f32x4 a = dc_load(&A[i][j]);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j + e < i) x = fmaf(-a[e], X[j + e], x);
      }
      X[i] = x;
      __builtin_amdgcn_sched_barrier(0);       // a row of A at a time in registers
    }
    if (is_v) {
      float* dst = up + item * DC * P + col;
#pragma unroll
      for (int i = 0; i < DC; ++i) dst[(long)i * P] = X[i];
    } else {
      float* dst = w + item * DC * N;
#pragma unroll
      for (int i = 0; i < DC; ++i) dst[dc_at(i, col - P, NT)] = X[i];
    }
  }
}

// grid (heads, P / 16, requests), four waves: a wave the sixteen tokens 16 wave .. of a chunk, and of the state the tiles
// of sixteen rows wave, wave + 4 in its accumulators.  The state's slice and U travel between the waves through LDS, value
// dim by value dim.  A chunk's operands are asked for while the chunk before is worked on.  spans5 [n][5] = (slot, first
// token, tokens, first chunk, chunks).  CHANNEL: a decay a key channel (see the kernel above).
template <int NT>
struct DeltaChunkOperands {
  static constexpr int TILES = (NT + 3) / 4;
  dc_f32x4 w[NT], q[NT], m[4], k[TILES][4], b_rows[TILES];
  float up[4], b[4], b_last;
};

template <int NT, bool CHANNEL>
__global__ void __launch_bounds__(256)
delta_chunk_walk_kernel(const float* __restrict__ q, const float* __restrict__ up, const float* __restrict__ w,
                        const float* __restrict__ kt, const float* __restrict__ m, const float* __restrict__ b,
                        const int32_t* __restrict__ spans5, const int32_t* __restrict__ positions, float* __restrict__ state,
                        long state_stride, long copy_elems, long tail_at, const float* __restrict__ conv_in, long conv_in_stride,
                        float* __restrict__ y, int heads, int kv_heads, int P, int taps) {
  typedef DeltaChunkOperands<NT> Ops;
  constexpr int N = 16 * NT, TILES = Ops::TILES;
  __shared__ __align__(16) float Sl[16][N + 4];
  __shared__ __align__(16) float Ul[16][DC + 4];
  const int h = blockIdx.x, kh = h / (heads / kv_heads), p0 = 16 * blockIdx.y;
  const int32_t* span = spans5 + 5 * blockIdx.z;
  const int slot = span[0], first = span[1], count = span[2], chunk0 = span[3], n_chunks = span[4];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g4 = lane >> 4;
  const int start = positions[first], channels = 2 * kv_heads * N + heads * P;
  const float* from = rec_copy_before(state, state_stride, copy_elems, slot, start);
  float* to = rec_copy_behind(state, state_stride, copy_elems, slot, start + count - 1);
  const long s_at = (long)h * N * P + (long)(p0 + r) * N + 4 * g4;
  dc_f32x4 S[TILES];
#pragma unroll
  for (int tt = 0; tt < TILES; ++tt) {
    S[tt] = dc_f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    const int tile = wave + 4 * tt;
    if (tile < NT) {
      S[tt] = dc_load(from + s_at + 16 * tile);
      *reinterpret_cast<dc_f32x4*>(&Sl[r][16 * tile + 4 * g4]) = S[tt];
    }
  }
  auto fetch = [&](Ops& o, int c) {
    const long item = (long)(chunk0 + c) * heads + h;
    const float* wr = w + item * DC * N + (wave * NT * 64 + lane) * 4;
    const float* qr = q + (CHANNEL ? item : (long)(chunk0 + c) * kv_heads + kh) * DC * N + (wave * NT * 64 + lane) * 4;
#pragma unroll
    for (int i = 0; i < NT; ++i) { o.w[i] = dc_load(wr + 256 * i); o.q[i] = dc_load(qr + 256 * i); }
    const float* mr = m + item * DC * DC + (wave * 4 * 64 + lane) * 4;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i <= wave) o.m[i] = dc_load(mr + 256 * i);
#pragma unroll
    for (int tt = 0; tt < TILES; ++tt)
      if (wave + 4 * tt < NT) {
        const float* kr = kt + item * N * DC + ((wave + 4 * tt) * 4 * 64 + lane) * 4;
#pragma unroll
        for (int i = 0; i < 4; ++i) o.k[tt][i] = dc_load(kr + 256 * i);
        if (CHANNEL) o.b_rows[tt] = dc_load(b + item * N + 16 * (wave + 4 * tt) + 4 * g4);
      }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o.up[e] = up[(item * DC + 16 * wave + 4 * g4 + e) * P + p0 + r];
      if (!CHANNEL) o.b[e] = b[item * DC + 16 * wave + 4 * g4 + e];
    }
    if (!CHANNEL) o.b_last = b[item * DC + DC - 1];
  };
  auto work = [&](const Ops& o, int c) {
    // two halves of the sum over the state's rows, two products: four chains
    dc_f32x4 ws[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}}, qs[2] = {ws[0], ws[0]};
    dc_f32x4 s[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) s[i] = dc_load(&Sl[r][16 * i + 4 * g4]);
#pragma unroll
    for (int i = 0; i < NT / 2; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        DC_MFMA(ws[0], o.w[i], s[i], j);
        DC_MFMA(qs[0], o.q[i], s[i], j);
        DC_MFMA(ws[1], o.w[NT / 2 + i], s[NT / 2 + i], j);
        DC_MFMA(qs[1], o.q[NT / 2 + i], s[NT / 2 + i], j);
      }
    dc_f32x4 mine, out;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      mine[e] = o.up[e] - (ws[0][e] + ws[1][e]);
      out[e] = (qs[0][e] + qs[1][e]) * (CHANNEL ? 1.0f : o.b[e]);
    }
    *reinterpret_cast<dc_f32x4*>(&Ul[r][16 * wave + 4 * g4]) = mine;
    __syncthreads();                       // every wave's part of U is there, and every wave has read the state
    dc_f32x4 all[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) all[i] = dc_load(&Ul[r][16 * i + 4 * g4]);
#pragma unroll
    for (int tt = 0; tt < TILES; ++tt)
#pragma unroll
      for (int e = 0; e < 4; ++e) S[tt][e] *= CHANNEL ? o.b_rows[tt][e] : o.b_last;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (i <= wave) DC_MFMA(out, o.m[i], all[i], j);
#pragma unroll
        for (int tt = 0; tt < TILES; ++tt)
          if (wave + 4 * tt < NT) DC_MFMA(S[tt], o.k[tt][i], all[i], j);
      }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = DC * c + 16 * wave + 4 * g4 + e;
      if (i < count) y[((long)(first + i) * heads + h) * P + p0 + r] = out[e];
    }
#pragma unroll
    for (int tt = 0; tt < TILES; ++tt)
      if (wave + 4 * tt < NT) *reinterpret_cast<dc_f32x4*>(&Sl[r][16 * (wave + 4 * tt) + 4 * g4]) = S[tt];
    __syncthreads();
  };
  Ops even, odd;
  fetch(even, 0);
  __syncthreads();
  for (int c = 0; c < n_chunks; c += 2) {
    if (c + 1 < n_chunks) fetch(odd, c + 1);
    work(even, c);
    if (c + 1 >= n_chunks) break;
    if (c + 2 < n_chunks) fetch(even, c + 2);
    work(odd, c + 1);
  }
#pragma unroll
  for (int tt = 0; tt < TILES; ++tt)
    if (wave + 4 * tt < NT) *reinterpret_cast<dc_f32x4*>(to + s_at + 16 * (wave + 4 * tt)) = S[tt];
  keep_conv_inputs(from + tail_at, to + tail_at, conv_in, conv_in_stride, first, count, channels, taps,
                   (blockIdx.x * gridDim.y + blockIdx.y) * 256 + threadIdx.x, gridDim.x * gridDim.y * 256);
}

// out[t, a] = (y[t, a] / sqrt(mean(y[t, a]^2) + eps)) gain act(gate[t, a]) head by head, act silu or sigmoid (GATE); the
// gain holds P numbers shared by the heads, or one for every channel (gain_per_head).  A wave a (token, head), or a block
// for heads of many values.
#define GATE_SILU 0
#define GATE_SIGMOID 1
__device__ inline float gate_act(float z, int kind) { return kind == GATE_SILU ? rec_silu(z) : rec_sigmoid(z); }
#define HN_KEPT 4
__global__ void __launch_bounds__(256)
head_norm_gate_kernel(const float* __restrict__ y, const float* __restrict__ gate, long gate_stride, const void* __restrict__ gain,
                      int gain_is_f32, int gain_per_head, float eps, elem_t* __restrict__ out, long items, int heads, int P,
                      int act) {
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int lane = threadIdx.x & 63, h = (int)(item % heads);
  const long t = item / heads;
  const float* src = y + item * P;
  const float* g = gate + t * gate_stride + (long)h * P;
  elem_t* dst = out + item * P;
  const int gain_at = gain_per_head ? h * P : 0;
  float kept[HN_KEPT], ss = 0.0f;
#pragma unroll
  for (int j = 0; j < HN_KEPT; ++j) {
    kept[j] = lane + 64 * j < P ? src[lane + 64 * j] : 0.0f;
    ss = fmaf(kept[j], kept[j], ss);
  }
  for (int i = lane + 64 * HN_KEPT; i < P; i += 64) ss = fmaf(src[i], src[i], ss);
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)P + eps);
#pragma unroll
  for (int j = 0; j < HN_KEPT; ++j) {
    const int i = lane + 64 * j;
    if (i < P) dst[i] = from_float(((kept[j] * inv) * load_vec(gain, gain_is_f32, gain_at + i)) * gate_act(g[i], act));
  }
  for (int i = lane + 64 * HN_KEPT; i < P; i += 64)
    dst[i] = from_float(((src[i] * inv) * load_vec(gain, gain_is_f32, gain_at + i)) * gate_act(g[i], act));
}

// The same for heads of 4 LANES values (16 to 256): LANES lanes a head, four values each.
template <int LANES>
__global__ void __launch_bounds__(256)
head_norm_gate_vec_kernel(const float* __restrict__ y, const float* __restrict__ gate, long gate_stride, const void* __restrict__ gain,
                          int gain_is_f32, int gain_per_head, float eps, elem_t* __restrict__ out, long items, int heads, int act) {
  constexpr int P = 4 * LANES;
  const long item = ((long)blockIdx.x * 256 + threadIdx.x) / LANES;
  const int e = 4 * (threadIdx.x % LANES);
  const bool active = item < items;
  const long it = active ? item : items - 1;
  const int h = (int)(it % heads);
  const float4 v = *reinterpret_cast<const float4*>(y + it * P + e);
  const float4 g = *reinterpret_cast<const float4*>(gate + it / heads * gate_stride + (long)h * P + e);
  const float4 w = load_vec4(gain, gain_is_f32, (gain_per_head ? h * P : 0) + e);
  float ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, v.w * v.w)));
#pragma unroll
  for (int off = LANES / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
  const float inv = 1.0f / sqrtf(ss / (float)P + eps);
  if (!active) return;
  const float o0 = ((v.x * inv) * w.x) * gate_act(g.x, act), o1 = ((v.y * inv) * w.y) * gate_act(g.y, act);
  const float o2 = ((v.z * inv) * w.z) * gate_act(g.z, act), o3 = ((v.w * inv) * w.w) * gate_act(g.w, act);
  elem_t* dst = out + it * P + e;
#if AXON_BF16
  *reinterpret_cast<uint2*>(dst) = make_uint2(pack2_bf16(o0, o1), pack2_bf16(o2, o3));
#else
  *reinterpret_cast<float4*>(dst) = make_float4(o0, o1, o2, o3);
#endif
}

// The same for heads of many values (all channels of a row normed together, say): a block a (token, head), G values a thread
// at a time, the first HN_KEPT of these and their gates kept in registers.
template <int G>
__global__ void __launch_bounds__(256)
head_norm_gate_wide_kernel(const float* __restrict__ y, const float* __restrict__ gate, long gate_stride, const void* __restrict__ gain,
                           int gain_is_f32, int gain_per_head, float eps, elem_t* __restrict__ out, int heads, int P, int act) {
  __shared__ float partial[256 / AXON_WAVE];
  const long item = blockIdx.x;
  const int h = (int)(item % heads), gain_at = gain_per_head ? h * P : 0;
  const float* src = y + item * P;
  const float* g = gate + item / heads * gate_stride + (long)h * P;
  elem_t* dst = out + item * P;
  auto load = [&](const float* p, float (&v)[G]) {
    if (G == 4) {
      const float4 q = *reinterpret_cast<const float4*>(p);
      v[0] = q.x; v[1 % G] = q.y; v[2 % G] = q.z; v[3 % G] = q.w;
    } else {
      v[0] = p[0];
    }
  };
  float kept[HN_KEPT][G], gates[HN_KEPT][G], ss = 0.0f;
#pragma unroll
  for (int j = 0; j < HN_KEPT; ++j) {
    const int i = G * (threadIdx.x + 256 * j);
    if (i >= P) break;
    load(src + i, kept[j]);
    load(g + i, gates[j]);
#pragma unroll
    for (int e = 0; e < G; ++e) ss = fmaf(kept[j][e], kept[j][e], ss);
  }
  for (int i = G * (threadIdx.x + 256 * HN_KEPT); i < P; i += G * 256) {
    float v[G];
    load(src + i, v);
#pragma unroll
    for (int e = 0; e < G; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float inv = 1.0f / sqrtf(block_sum_256(ss, partial) / (float)P + eps);
  auto store = [&](int i, const float (&v)[G], const float (&z)[G]) {
    float o[G];
#pragma unroll
    for (int e = 0; e < G; ++e) o[e] = ((v[e] * inv) * load_vec(gain, gain_is_f32, gain_at + i + e)) * gate_act(z[e], act);
#if AXON_BF16
    if (G == 4) *reinterpret_cast<uint2*>(dst + i) = make_uint2(pack2_bf16(o[0], o[1 % G]), pack2_bf16(o[2 % G], o[3 % G]));
#else
    if (G == 4) *reinterpret_cast<float4*>(dst + i) = make_float4(o[0], o[1 % G], o[2 % G], o[3 % G]);
#endif
    else dst[i] = from_float(o[0]);
  };
#pragma unroll
  for (int j = 0; j < HN_KEPT; ++j) {
    const int i = G * (threadIdx.x + 256 * j);
    if (i < P) store(i, kept[j], gates[j]);
  }
  for (int i = G * (threadIdx.x + 256 * HN_KEPT); i < P; i += G * 256) {
    float v[G], z[G];
    load(src + i, v);
    load(g + i, z);
    store(i, v, z);
  }
}

// delta_prepare for long steps and up to four taps: a wave a head of queries or keys or up to 256 value channels, over
// DP_TOKENS tokens in a row, whose inputs and weights stay in registers.  The same sums as the kernel above.
#define DP_TOKENS 8
template <int TAPS>
__global__ void __launch_bounds__(256)
delta_prepare_run_kernel(const float* __restrict__ in, long in_stride, const elem_t* __restrict__ w, const float* __restrict__ state,
                         long state_stride, long copy_elems, long tail_at, const int32_t* __restrict__ positions,
                         const int32_t* __restrict__ seq_rows, int beta_at, int decay_at, const void* __restrict__ a_log,
                         int a_log_is_f32, const void* __restrict__ dt_bias, int dt_bias_is_f32, float* __restrict__ u,
                         float* __restrict__ terms, int n_tokens, int heads, int kv_heads, int N, int P, float q_scale) {
  const int t0 = blockIdx.x * DP_TOKENS, t1 = min(t0 + DP_TOKENS, n_tokens), unit = blockIdx.y * 4 + (threadIdx.x >> 6),
            lane = threadIdx.x & 63;
  const int v_units = (heads * P + 255) / 256, channels = 2 * kv_heads * N + heads * P;
  if (unit > 2 * kv_heads + v_units) return;
  if (unit == 2 * kv_heads + v_units) {
    for (int i = lane; i < heads * (t1 - t0); i += 64) {
      const int t = t0 + i / heads, a = i % heads;
      const float* row = in + (long)t * in_stride;
      terms[((long)t * heads + a) * 2] = delta_decay(row, decay_at, a_log, a_log_is_f32, dt_bias, dt_bias_is_f32, a);
      terms[((long)t * heads + a) * 2 + 1] = rec_sigmoid(row[beta_at + a]);
    }
    return;
  }
  const bool is_v = unit >= 2 * kv_heads;
  const int c0 = is_v ? 2 * kv_heads * N + 256 * (unit - 2 * kv_heads) : unit * N, size = is_v ? min(256, channels - c0) : N;
  float wt[DP_KEPT][TAPS], past[DP_KEPT][TAPS];        // past[j][k]: the input k tokens before
  int c[DP_KEPT];
#pragma unroll
  for (int j = 0; j < DP_KEPT; ++j) {
    c[j] = c0 + min(lane + 64 * j, size - 1);
#pragma unroll
    for (int k = 0; k < TAPS; ++k) wt[j][k] = to_float(w[(long)c[j] * TAPS + k]);
  }
  int slot_before = -1;
  for (int t = t0; t < t1; ++t) {
    const int slot = seq_rows[t];
    const float* row = in + (long)t * in_stride;
    if (slot != slot_before) {
      const int inside = rec_inside(seq_rows, t, TAPS - 1);
      const float* kept = rec_copy_before(state, state_stride, copy_elems, slot, positions[t] - inside) + tail_at;
#pragma unroll
      for (int j = 0; j < DP_KEPT; ++j)
#pragma unroll
        for (int k = 1; k < TAPS; ++k)
          past[j][k] = k <= inside ? row[c[j] - (long)k * in_stride] : kept[(long)(TAPS - 1 - (k - inside)) * channels + c[j]];
      slot_before = slot;
    }
    float v[DP_KEPT], ss = 0.0f;
#pragma unroll
    for (int j = 0; j < DP_KEPT; ++j) {
      v[j] = 0.0f;
      if (64 * j >= size) continue;                    // the whole wave
      past[j][0] = row[c[j]];
      float acc = 0.0f;
#pragma unroll
      for (int k = 0; k < TAPS; ++k) acc = fmaf(wt[j][k], past[j][TAPS - 1 - k], acc);
#pragma unroll
      for (int k = TAPS - 1; k > 0; --k) past[j][k] = past[j][k - 1];
      v[j] = lane + 64 * j < size ? rec_silu(acc) : 0.0f;
      ss = fmaf(v[j], v[j], ss);
    }
    const float inv = is_v ? 1.0f : (1.0f / sqrtf(wave_sum(ss) + 1e-6f)) * (unit < kv_heads ? q_scale : 1.0f);
    float* dst = u + (long)t * channels + c0;
#pragma unroll
    for (int j = 0; j < DP_KEPT; ++j)
      if (lane + 64 * j < size) dst[lane + 64 * j] = v[j] * inv;
  }
}

}  // namespace

extern "C" int axk_delta_prepare(const float* in, long in_stride, const void* w, int taps, const float* state, long state_stride,
                                 long copy_elems, long tail_at, const int32_t* positions, const int32_t* seq_rows, int beta_at,
                                 int decay_at, const void* a_log, int a_log_is_f32, const void* dt_bias, int dt_bias_is_f32, float* u,
                                 float* terms, int n_tokens, int heads, int kv_heads, int N, int P, float q_scale, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && N > 0 && N <= 256 && P > 0 && taps >= 1,
              "delta_prepare: bad sizes T=%d heads=%d kv heads=%d keys=%d (at most 256) values=%d taps=%d", n_tokens, heads, kv_heads,
              N, P, taps);
  const long channels = 2L * kv_heads * N + (long)heads * P;
  AXK_REQUIRE(in_stride >= channels && beta_at >= 0 && beta_at + heads <= in_stride &&
              (a_log == nullptr || (decay_at >= 0 && decay_at + heads <= in_stride)),
              "delta_prepare: the parts do not fit rows of %ld", in_stride);
  AXK_REQUIRE(tail_at >= 0 && copy_elems >= tail_at + (taps - 1) * channels && state_stride >= 2 * copy_elems,
              "delta_prepare: a state row of %ld floats does not hold two copies of %ld with %d x %ld kept inputs from %ld",
              state_stride, copy_elems, taps - 1, channels, tail_at);
  if (n_tokens == 0) return 0;
  if (n_tokens >= 256 && taps <= 4) {
    const dim3 grid(ceil_div(n_tokens, DP_TOKENS), ceil_div(2 * kv_heads + ceil_div(heads * P, 256) + 1, 4));
#define DP_RUN(TAPS)                                                                                                            \
  delta_prepare_run_kernel<TAPS><<<grid, 256, 0, (hipStream_t)stream>>>(in, in_stride, (const elem_t*)w, state, state_stride, \
      copy_elems, tail_at, positions, seq_rows, beta_at, decay_at, a_log, a_log_is_f32, dt_bias, dt_bias_is_f32, u, terms,      \
      n_tokens, heads, kv_heads, N, P, q_scale)
    if (taps == 1) DP_RUN(1); else if (taps == 2) DP_RUN(2); else if (taps == 3) DP_RUN(3); else DP_RUN(4);
#undef DP_RUN
    AXK_LAUNCH_CHECK("delta_prepare");
    return 0;
  }
  delta_prepare_kernel<<<dim3(n_tokens, ceil_div(2 * kv_heads + heads + 1, 4)), 256, 0, (hipStream_t)stream>>>(
      in, in_stride, (const elem_t*)w, taps, state, state_stride, copy_elems, tail_at, positions, seq_rows, beta_at, decay_at, a_log,
      a_log_is_f32, dt_bias, dt_bias_is_f32, u, terms, heads, kv_heads, N, P, q_scale);
  AXK_LAUNCH_CHECK("delta_prepare");
  return 0;
}

extern "C" int axk_delta_scan(const float* u, const float* terms, const float* decay, float* state, long state_stride, long copy_elems, long tail_at,
                              const int32_t* spans, int n_spans, const int32_t* positions, const int32_t* seq_rows,
                              const float* conv_in, long conv_in_stride, float* y, int heads, int kv_heads, int N, int P, int taps,
                              void* stream) {
  AXK_REQUIRE(n_spans >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && N > 0 && N <= 256 && P > 0 && taps >= 1,
              "delta_scan: bad sizes spans=%d heads=%d kv heads=%d keys=%d (at most 256) values=%d taps=%d", n_spans, heads, kv_heads,
              N, P, taps);
  const long channels = 2L * kv_heads * N + (long)heads * P;
  AXK_REQUIRE(tail_at >= (long)heads * N * P && copy_elems >= tail_at + (taps - 1) * channels && state_stride >= 2 * copy_elems &&
              conv_in_stride >= channels,
              "delta_scan: a state row of %ld floats does not hold two copies of %ld (%d x %d x %d, then %d x %ld from %ld)", state_stride,
              copy_elems, heads, N, P, taps - 1, channels, tail_at);
  AXK_REQUIRE((spans != nullptr || seq_rows != nullptr) && positions != nullptr, "delta_scan: neither spans nor slots, or no positions");
  if (n_spans == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = N % 4 == 0 && channels % 4 == 0 && copy_elems % 4 == 0 && state_stride % 4 == 0 && ((uintptr_t)u & 15) == 0 &&
                   ((uintptr_t)state & 15) == 0 && ((uintptr_t)decay & 15) == 0;
#define DELTA_ARGS u, terms, decay, state, state_stride, copy_elems, tail_at, spans, positions, seq_rows, conv_in, conv_in_stride, y, heads, \
                   kv_heads, N, P, taps
#define DELTA_LAUNCH(LK, OWN)                                                                    \
  {                                                                                              \
    const dim3 grid(n_spans, heads, ceil_div(P, REC_THREADS / LK));                              \
    if (decay == nullptr) {                                                                      \
      if (vec) delta_scan_kernel<LK, OWN, true, false><<<grid, REC_THREADS, 0, s>>>(DELTA_ARGS); \
      else delta_scan_kernel<LK, OWN, false, false><<<grid, REC_THREADS, 0, s>>>(DELTA_ARGS);    \
    } else if (vec) delta_scan_kernel<LK, OWN, true, true><<<grid, REC_THREADS, 0, s>>>(DELTA_ARGS); \
    else delta_scan_kernel<LK, OWN, false, true><<<grid, REC_THREADS, 0, s>>>(DELTA_ARGS);       \
  }
  REC_BY_ROWS(N, DELTA_LAUNCH)
#undef DELTA_LAUNCH
#undef DELTA_ARGS
  AXK_LAUNCH_CHECK("delta_scan");
  return 0;
}

// 1 where axk_delta_chunked takes these sizes.
extern "C" int axk_delta_chunked_ok(int kv_heads, int heads, int N, int P) {
  return (N == 32 || N == 64 || N == 96 || N == 128) && P % 16 == 0 && P / 16 <= 65535 && heads > 0 && kv_heads > 0;
}

// The floats of workspace that axk_delta_chunked wants for this many chunks.
extern "C" long axk_delta_chunked_workspace(int n_chunks, int heads, int N, int P) {
  return (long)n_chunks * heads * (DC * (3L * N + P + DC) + (N > DC ? N : DC));
}

extern "C" int axk_delta_chunked(const float* u, const float* terms, const float* decay, float* state, long state_stride, long copy_elems, long tail_at,
                                 const int32_t* chunks, int n_chunks, const int32_t* spans5, int n_spans, const int32_t* positions,
                                 const float* conv_in, long conv_in_stride, float* y, int heads, int kv_heads, int N, int P, int taps,
                                 float* work, long work_floats, void* stream) {
  AXK_REQUIRE(n_spans >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && taps >= 1 && axk_delta_chunked_ok(kv_heads, heads, N, P),
              "delta_chunked: bad sizes spans=%d heads=%d kv heads=%d keys=%d values=%d taps=%d", n_spans, heads, kv_heads, N, P, taps);
  const long channels = 2L * kv_heads * N + (long)heads * P;
  AXK_REQUIRE(tail_at >= (long)heads * N * P && copy_elems >= tail_at + (taps - 1) * channels && state_stride >= 2 * copy_elems &&
              conv_in_stride >= channels,
              "delta_chunked: a state row of %ld floats does not hold two copies of %ld (%d x %d x %d, then %d x %ld from %ld)",
              state_stride, copy_elems, heads, N, P, taps - 1, channels, tail_at);
  AXK_REQUIRE(copy_elems % 4 == 0 && state_stride % 4 == 0 && ((uintptr_t)u & 15) == 0 && ((uintptr_t)state & 15) == 0 &&
              ((uintptr_t)work & 15) == 0 && ((uintptr_t)decay & 15) == 0, "delta_chunked: rows are not 16-byte aligned");
  AXK_REQUIRE(n_chunks >= n_spans && n_chunks <= 65535 && n_spans <= 65535, "delta_chunked: %d chunks of %d requests", n_chunks, n_spans);
  AXK_REQUIRE(work != nullptr && work_floats >= axk_delta_chunked_workspace(n_chunks, heads, N, P), "delta_chunked: a workspace of %ld floats",
              work_floats);
  if (n_spans == 0) return 0;
  const long items = (long)n_chunks * heads;
  float* up = work;
  float* w = up + items * DC * P;
  float* kt = w + items * DC * N;
  float* m = kt + items * DC * N;
  float* q = m + items * DC * DC;
  float* b = q + (decay ? items : (long)n_chunks * kv_heads) * DC * N;
  hipStream_t s = (hipStream_t)stream;
#define DC_WALK(NT, CHANNEL)                                                                                                    \
  delta_chunk_walk_kernel<NT, CHANNEL><<<dim3(heads, P / 16, n_spans), 256, 0, s>>>(                                            \
      q, up, w, kt, m, b, spans5, positions, state, state_stride, copy_elems, tail_at, conv_in, conv_in_stride, y, heads, kv_heads, P, taps)
#define DC_LAUNCH(NT)                                                                                                            \
  if (decay == nullptr) {                                                                                                        \
    delta_chunk_terms_kernel<NT><<<dim3(heads, n_chunks), 256, 0, s>>>(u, terms, chunks, heads, kv_heads, P, up, w, kt, m, q, b);\
    DC_WALK(NT, false);                                                                                                          \
  } else {                                                                                                                       \
    delta_chunk_channel_terms_kernel<NT><<<dim3(heads, n_chunks), 256, 0, s>>>(u, terms, decay, chunks, heads, kv_heads, P, up, w, kt, m, \
                                                                              q, b);                                             \
    DC_WALK(NT, true);                                                                                                           \
  }
  if (N == 32) { DC_LAUNCH(2) } else if (N == 64) { DC_LAUNCH(4) } else if (N == 96) { DC_LAUNCH(6) } else { DC_LAUNCH(8) }
#undef DC_LAUNCH
#undef DC_WALK
  AXK_LAUNCH_CHECK("delta_chunked");
  return 0;
}

extern "C" int axk_head_norm_gate(const float* y, const float* gate, long gate_stride, const void* gain, int gain_is_f32,
                                  int gain_per_head, int act, float eps, void* out, int n_tokens, int heads, int P, void* stream) {
  AXK_REQUIRE(n_tokens >= 0 && heads > 0 && P > 0 && gate_stride >= (long)heads * P,
              "head_norm_gate: bad sizes T=%d heads=%d values=%d gate rows of %ld", n_tokens, heads, P, gate_stride);
  AXK_REQUIRE(act == GATE_SILU || act == GATE_SIGMOID, "head_norm_gate: unknown gate %d", act);
  if (n_tokens == 0) return 0;
  const long items = (long)n_tokens * heads;
  const bool vec = gate_stride % 4 == 0 && (((uintptr_t)y | (uintptr_t)gate | (uintptr_t)gain | (uintptr_t)out) & 15) == 0;
#define HN_VEC(LANES)                                                                                                       \
  if (vec && P == 4 * LANES) {                                                                                              \
    head_norm_gate_vec_kernel<LANES><<<(unsigned)((items * LANES + 255) / 256), 256, 0, (hipStream_t)stream>>>(             \
        y, gate, gate_stride, gain, gain_is_f32, gain_per_head, eps, (elem_t*)out, items, heads, act);                         \
    AXK_LAUNCH_CHECK("head_norm_gate");                                                                                     \
    return 0;                                                                                                               \
  }
  HN_VEC(4) HN_VEC(8) HN_VEC(16) HN_VEC(32) HN_VEC(64)
#undef HN_VEC
  if (P > 512) {
    auto kernel = vec && P % 4 == 0 ? head_norm_gate_wide_kernel<4> : head_norm_gate_wide_kernel<1>;
    kernel<<<(unsigned)items, 256, 0, (hipStream_t)stream>>>(y, gate, gate_stride, gain, gain_is_f32, gain_per_head, eps, (elem_t*)out,
                                                             heads, P, act);
    AXK_LAUNCH_CHECK("head_norm_gate");
    return 0;
  }
  head_norm_gate_kernel<<<(unsigned)((items + 3) / 4), 256, 0, (hipStream_t)stream>>>(y, gate, gate_stride, gain, gain_is_f32,
                                                                                     gain_per_head, eps, (elem_t*)out, items, heads, P, act);
  AXK_LAUNCH_CHECK("head_norm_gate");
  return 0;
}
