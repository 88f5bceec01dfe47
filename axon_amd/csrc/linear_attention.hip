// Linear attention with a constant decay a head ("lightning attention"): per request and head a state matrix S [N, P],
//
//   S_t = decay_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,
//
// q, k and v (and all sums) 32-bit, taken through silu first.  A copy of the state row (see recurrence.h) holds the
// heads' states [heads][P][N] and nothing else.
#include "api.h"
#include "recurrence.h"

namespace {

// silu in place over the first `columns` numbers of every row (rows `stride` apart), for steps whose operands are read
// more than once.
__global__ void __launch_bounds__(256)
silu_rows_kernel(float* __restrict__ rows, long stride, int columns, int vec) {
  float* row = rows + (long)blockIdx.y * stride;
  const int i = (vec ? 4 : 1) * (blockIdx.x * 256 + threadIdx.x);
  if (i >= columns) return;
  if (vec) {
    float4 v = *reinterpret_cast<float4*>(row + i);
    v.x = rec_silu(v.x); v.y = rec_silu(v.y); v.z = rec_silu(v.z); v.w = rec_silu(v.w);
    *reinterpret_cast<float4*>(row + i) = v;
  } else {
    row[i] = rec_silu(row[i]);
  }
}

// The walk.  grid (requests of the step, heads, blocks of value dims); LK lanes share a value dim, OWN rows of the state
// a lane; the operands of AHEAD tokens are asked for while those before them are worked on.
template <int OWN, int AHEAD>
struct LightningOperands {
  float q[AHEAD][OWN], k[AHEAD][OWN], v[AHEAD];
};

template <int LK, int OWN, bool VEC>
__global__ void __launch_bounds__(REC_THREADS)
lightning_scan_kernel(const float* __restrict__ rows, long stride, int q_at, int k_at, int v_at, int silu,
                      const float* __restrict__ decay, float* __restrict__ state, long state_stride, long copy_elems,
                      const int32_t* __restrict__ spans, const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_rows,
                      float* __restrict__ y, int heads, int N, int P) {
  constexpr int AHEAD = OWN >= 16 ? 2 : 4;
  const RecStretch s = rec_stretch(nullptr, spans, seq_rows, blockIdx.x);
  const int h = blockIdx.y, ns = threadIdx.x % LK, n0 = ns * OWN;
  const int p = blockIdx.z * (REC_THREADS / LK) + threadIdx.x / LK;
  const bool has_p = p < P;
  const int start = positions[s.first];
  const float* from = rec_copy_before(state, state_stride, copy_elems, s.slot, start);
  float* to = rec_copy_behind(state, state_stride, copy_elems, s.slot, start + s.count - 1);
  const long s_at = (long)h * N * P + (long)p * N;
  const float d = decay[h];
  float S[OWN];
  if (has_p) rec_load<OWN, VEC>(S, from + s_at, n0, N);
  else {
#pragma unroll
    for (int i = 0; i < OWN; ++i) S[i] = 0.0f;
  }
  const int last = s.first + s.count;
  const long q_col = q_at + (long)h * N, k_col = k_at + (long)h * N, v_col = v_at + (long)h * P + (has_p ? p : 0);
  typedef LightningOperands<OWN, AHEAD> Ops;
  auto fetch = [&](Ops& o, int t0) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const float* row = rows + (long)min(t0 + a, last - 1) * stride;        // behind the last token: the last again, not used
      rec_load<OWN, VEC>(o.q[a], row + q_col, n0, N);
      rec_load<OWN, VEC>(o.k[a], row + k_col, n0, N);
      o.v[a] = row[v_col];
    }
  };
  auto work = [&](Ops& o, int t0) {
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      if (t0 + a >= last) break;
      if (silu) {                                          // rows beyond N read as zeros, and silu(0) is 0
        o.v[a] = rec_silu(o.v[a]);
#pragma unroll
        for (int i = 0; i < OWN; ++i) { o.q[a][i] = rec_silu(o.q[a][i]); o.k[a][i] = rec_silu(o.k[a][i]); }
      }
      float part = 0.0f;
#pragma unroll
      for (int i = 0; i < OWN; ++i) {
        S[i] = fmaf(o.k[a][i], o.v[a], d * S[i]);
        part = fmaf(S[i], o.q[a][i], part);
      }
      part = rec_row_sum<LK>(part);
      if (ns == 0 && has_p) y[((long)(t0 + a) * heads + h) * P + p] = part;
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
}

// Long stretches in chunks of up to 64 tokens, on the 32-bit matrix cores, everything but the fold side by side.  With
// i, j = 0, 1, ... inside a chunk of C tokens that finds the state I:
//   ends    E = sum_j decay^(C-1-j) k_j v_j^T                        per (chunk, head)
//   fold    I_0 = the request's state, I_(c+1) = decay^C I_c + E_c   element by element (I_c is left in E_c's place)
//   outputs o_i = decay^(i+1) I^T q_i + sum_(j<=i) decay^(i-j) (q_i . k_j) v_j
// Sixteen k of a product are four chained instructions: lane l holds rows l % 16 at k = 4 (l / 16) .. + 3 of either
// operand, instruction j takes their j-th; of the result it holds column l % 16 of rows 4 (l / 16) .. + 3.
#define LC 64
typedef __attribute__((ext_vector_type(4))) float lc_f32x4;
__device__ inline lc_f32x4 lc_load(const float* p) { return *reinterpret_cast<const lc_f32x4*>(p); }
#define LC_MFMA(acc, a, b, j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32((a)[j], (b)[j], acc, 0, 0, 0)

// powers[i] = decay^i, i <= LC, in LDS: by repeated squaring, so an early power does not gather the rounding of a long chain.
__device__ inline void lc_powers(float* powers, float d, int tid) {
  if (tid <= LC) {
    float r = 1.0f, b = d;
    for (int e = tid; e > 0; e >>= 1) {
      if (e & 1) r *= b;
      b *= b;
    }
    powers[tid] = r;
  }
}

// grid (heads, chunks, row tiles of 64 keys): a wave sixteen rows n of the state, all value dims, two tiles of them at a time
// (two chains), the next two asked for while these are multiplied.
__global__ void __launch_bounds__(256)
lightning_ends_kernel(const float* __restrict__ rows, long stride, int k_at, int v_at, const float* __restrict__ decay,
                      const int32_t* __restrict__ chunks, float* __restrict__ ends, int heads, int N, int P) {
  __shared__ float powers[LC + 1];
  const int h = blockIdx.x, first = chunks[2 * blockIdx.y], count = chunks[2 * blockIdx.y + 1];
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, r = lane & 15, g4 = lane >> 4;
  lc_powers(powers, decay[h], tid);
  __syncthreads();
  const int n0 = 64 * blockIdx.z + 16 * wave;
  if (n0 >= N) return;
  lc_f32x4 k[LC / 16];
  const float* vcol = rows + v_at + (long)h * P + r;
  int at[LC / 16][4];
#pragma unroll
  for (int c = 0; c < LC / 16; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = 16 * c + 4 * g4 + e;
      at[c][e] = first + min(j, count - 1);
      k[c][e] = j < count ? rows[at[c][e] * stride + k_at + (long)h * N + n0 + r] * powers[count - 1 - j] : 0.0f;
    }
  float* dst = ends + ((long)blockIdx.y * heads + h) * N * P + n0 + 4 * g4;
  lc_f32x4 even[2][LC / 16], odd[2][LC / 16];
  auto fetch = [&](lc_f32x4 (&v)[2][LC / 16], int p0) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
      if (p0 + 16 * i < P) {
#pragma unroll
        for (int c = 0; c < LC / 16; ++c)
#pragma unroll
          for (int e = 0; e < 4; ++e) v[i][c][e] = vcol[at[c][e] * stride + p0 + 16 * i];
      }
  };
  auto work = [&](const lc_f32x4 (&v)[2][LC / 16], int p0) {
    lc_f32x4 acc[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}};
#pragma unroll
    for (int c = 0; c < LC / 16; ++c)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 2; ++i) LC_MFMA(acc[i], k[c], v[i][c], j);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      if (p0 + 16 * i < P) *reinterpret_cast<lc_f32x4*>(dst + (long)(p0 + 16 * i + r) * N) = acc[i];
  };
#pragma unroll
  for (int i = 0; i < 2; ++i)                      // a tile beyond P holds zeros, then whatever was last there: not stored
#pragma unroll
    for (int c = 0; c < LC / 16; ++c) even[i][c] = odd[i][c] = lc_f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  fetch(even, 0);
  for (int p0 = 0; p0 < P; p0 += 64) {
    if (p0 + 32 < P) fetch(odd, p0 + 32);
    work(even, p0);
    if (p0 + 32 >= P) break;
    if (p0 + 64 < P) fetch(even, p0 + 64);
    work(odd, p0 + 32);
  }
}

// spans5 [n][5] = (slot, first token, tokens, first chunk, chunks); an element of the state a thread.
__global__ void __launch_bounds__(256)
lightning_fold_kernel(float* __restrict__ ends, const float* __restrict__ decay, const int32_t* __restrict__ chunks,
                      const int32_t* __restrict__ spans5, float* __restrict__ state, long state_stride, long copy_elems,
                      const int32_t* __restrict__ positions, int heads, int N, int P) {
  __shared__ float powers[LC + 1];
  const int h = blockIdx.z;
  lc_powers(powers, decay[h], threadIdx.x);
  __syncthreads();
  const int32_t* span = spans5 + 5 * blockIdx.x;
  const int slot = span[0], first = span[1], count = span[2], chunk0 = span[3], n_chunks = span[4];
  const long i = (long)blockIdx.y * 256 + threadIdx.x, size = (long)N * P, all = heads * size;
  if (i >= size) return;
  const int start = positions[first];
  float I = rec_copy_before(state, state_stride, copy_elems, slot, start)[h * size + i];
  float* mine = ends + (long)chunk0 * all + h * size + i;
  for (int c = 0; c < n_chunks; c += 8) {
    float e[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) e[j] = mine[(long)min(c + j, n_chunks - 1) * all];
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (c + j < n_chunks) {
        mine[(long)(c + j) * all] = I;
        I = fmaf(powers[chunks[2 * (chunk0 + c + j) + 1]], I, e[j]);
      }
  }
  rec_copy_behind(state, state_stride, copy_elems, slot, start + count - 1)[h * size + i] = I;
}

// grid (heads, chunks, blocks of VT tiles of sixteen value dims): a wave the sixteen tokens 16 wave .. of the chunk.  The
// products k_j . q_i are made transposed (rows j, column i), which is how the weighted sum over j wants its first operand.
#define LC_VT 4
struct LcOperands {
  lc_f32x4 q, k[LC / 16], s[LC_VT];
};

__global__ void __launch_bounds__(256)
lightning_outputs_kernel(const float* __restrict__ rows, long stride, int q_at, int k_at, int v_at, const float* __restrict__ decay,
                         const int32_t* __restrict__ chunks, const float* __restrict__ states, float* __restrict__ y, int heads, int N,
                         int P) {
  __shared__ float powers[LC + 1];
  const int h = blockIdx.x, first = chunks[2 * blockIdx.y], count = chunks[2 * blockIdx.y + 1];
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, r = lane & 15, g4 = lane >> 4;
  lc_powers(powers, decay[h], tid);
  __syncthreads();
  if (16 * wave >= count) return;
  const int nt = N / 16, p_first = 16 * LC_VT * blockIdx.z, tiles = min(LC_VT, (P - p_first) / 16);
  const float* q = rows + (long)(first + min(16 * wave + r, count - 1)) * stride + q_at + (long)h * N + 4 * g4;
  const float* I = states + (((long)blockIdx.y * heads + h) * P + p_first + r) * N + 4 * g4;
  const float* k[LC / 16];
#pragma unroll
  for (int c = 0; c < LC / 16; ++c) k[c] = rows + (long)(first + min(16 * c + r, count - 1)) * stride + k_at + (long)h * N + 4 * g4;
  lc_f32x4 m[LC / 16], out[LC_VT];
#pragma unroll
  for (int c = 0; c < LC / 16; ++c) m[c] = lc_f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
  for (int v = 0; v < LC_VT; ++v) out[v] = lc_f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  auto fetch = [&](LcOperands& o, int t) {
    o.q = lc_load(q + 16 * t);
#pragma unroll
    for (int c = 0; c < LC / 16; ++c)
      if (c <= wave) o.k[c] = lc_load(k[c] + 16 * t);
#pragma unroll
    for (int v = 0; v < LC_VT; ++v)
      if (v < tiles) o.s[v] = lc_load(I + (long)16 * v * N + 16 * t);
  };
  auto work = [&](const LcOperands& o) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int c = 0; c < LC / 16; ++c)
        if (c <= wave) LC_MFMA(m[c], o.k[c], o.q, j);
#pragma unroll
      for (int v = 0; v < LC_VT; ++v)
        if (v < tiles) LC_MFMA(out[v], o.q, o.s[v], j);
    }
  };
  LcOperands even, odd;
  fetch(even, 0);
  for (int t = 0; t < nt; t += 2) {
    if (t + 1 < nt) fetch(odd, t + 1);
    work(even);
    if (t + 1 >= nt) break;
    if (t + 2 < nt) fetch(even, t + 2);
    work(odd);
  }
  // the values of the chunk's tokens 16 c .., as the weighted sum's second operand
  lc_f32x4 v0[LC_VT], v1[LC_VT];
  auto values = [&](lc_f32x4 (&vf)[LC_VT], int c) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float* vrow = rows + (long)(first + min(16 * c + 4 * g4 + e, count - 1)) * stride + v_at + (long)h * P + p_first + r;
#pragma unroll
      for (int v = 0; v < LC_VT; ++v)
        if (v < tiles) vf[v][e] = vrow[16 * v];
    }
  };
  values(v0, 0);
  // the state's share of token i is decayed i + 1 times; the result's lane holds rows 4 g4 + e, the products' column r
#pragma unroll
  for (int v = 0; v < LC_VT; ++v)
#pragma unroll
    for (int e = 0; e < 4; ++e) out[v][e] *= powers[16 * wave + 4 * g4 + e + 1];
  const int i = 16 * wave + r;
#pragma unroll
  for (int c = 0; c < LC / 16; ++c)
    if (c <= wave) {
      lc_f32x4 (&now)[LC_VT] = c % 2 ? v1 : v0;
      if (c + 1 < LC / 16 && c + 1 <= wave) values(c % 2 ? v0 : v1, c + 1);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = 16 * c + 4 * g4 + e;
        m[c][e] = j <= i ? m[c][e] * powers[max(i - j, 0)] : 0.0f;
      }
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int v = 0; v < LC_VT; ++v)
          if (v < tiles) LC_MFMA(out[v], m[c], now[v], j);
    }
#pragma unroll
  for (int v = 0; v < LC_VT; ++v)
    if (v < tiles)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * wave + 4 * g4 + e;
        if (t < count) y[((long)(first + t) * heads + h) * P + p_first + 16 * v + r] = out[v][e];
      }
}

}  // namespace

extern "C" int axk_silu_rows(float* rows, long stride, int columns, int n_rows, void* stream) {
  AXK_REQUIRE(n_rows >= 0 && columns > 0 && stride >= columns, "silu_rows: %d columns of rows of %ld", columns, stride);
  if (n_rows == 0) return 0;
  AXK_REQUIRE(n_rows <= 65535, "silu_rows: %d rows in one step (at most 65535)", n_rows);
  const int vec = columns % 4 == 0 && stride % 4 == 0 && ((uintptr_t)rows & 15) == 0;
  silu_rows_kernel<<<dim3(ceil_div(columns, vec ? 1024 : 256), n_rows), 256, 0, (hipStream_t)stream>>>(rows, stride, columns, vec);
  AXK_LAUNCH_CHECK("silu_rows");
  return 0;
}

static int lightning_sizes_ok(const char* what, int heads, int N, int P, long stride, int q_at, int k_at, int v_at, long state_stride,
                              long copy_elems) {
  AXK_REQUIRE(heads > 0 && N > 0 && N <= 256 && P > 0 && heads <= 65535, "%s: bad sizes heads=%d keys=%d (at most 256) values=%d", what,
              heads, N, P);
  AXK_REQUIRE(q_at >= 0 && k_at >= 0 && v_at >= 0 && q_at + (long)heads * N <= stride && k_at + (long)heads * N <= stride &&
              v_at + (long)heads * P <= stride, "%s: the parts do not fit rows of %ld", what, stride);
  AXK_REQUIRE(copy_elems >= (long)heads * N * P && state_stride >= 2 * copy_elems,
              "%s: a state row of %ld floats does not hold two copies of %d x %d x %d", what, state_stride, heads, N, P);
  return 0;
}

extern "C" int axk_lightning_scan(const float* rows, long stride, int q_at, int k_at, int v_at, int silu, const float* decay, float* state,
                                  long state_stride, long copy_elems, const int32_t* spans, int n_spans, const int32_t* positions,
                                  const int32_t* seq_rows, float* y, int heads, int N, int P, void* stream) {
  const int rc = lightning_sizes_ok("lightning_scan", heads, N, P, stride, q_at, k_at, v_at, state_stride, copy_elems);
  if (rc != 0) return rc;
  AXK_REQUIRE(n_spans >= 0 && (spans != nullptr || seq_rows != nullptr) && positions != nullptr,
              "lightning_scan: neither spans nor slots, or no positions");
  if (n_spans == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = N % 4 == 0 && stride % 4 == 0 && q_at % 4 == 0 && k_at % 4 == 0 && copy_elems % 4 == 0 && state_stride % 4 == 0 &&
                   ((uintptr_t)rows & 15) == 0 && ((uintptr_t)state & 15) == 0;
#define LIGHTNING_ARGS rows, stride, q_at, k_at, v_at, silu, decay, state, state_stride, copy_elems, spans, positions, seq_rows, y, heads, N, P
#define LIGHTNING_LAUNCH(LK, OWN)                                                                \
  {                                                                                              \
    const dim3 grid(n_spans, heads, ceil_div(P, REC_THREADS / LK));                              \
    if (vec) lightning_scan_kernel<LK, OWN, true><<<grid, REC_THREADS, 0, s>>>(LIGHTNING_ARGS);  \
    else lightning_scan_kernel<LK, OWN, false><<<grid, REC_THREADS, 0, s>>>(LIGHTNING_ARGS);     \
  }
  REC_BY_ROWS(N, LIGHTNING_LAUNCH)
#undef LIGHTNING_LAUNCH
#undef LIGHTNING_ARGS
  AXK_LAUNCH_CHECK("lightning_scan");
  return 0;
}

// 1 where axk_lightning_chunked takes these sizes (rows whose parts lie at multiples of four floats).
extern "C" int axk_lightning_chunked_ok(int heads, int N, int P, long stride, int q_at, int k_at) {
  return heads > 0 && N > 0 && N <= 256 && N % 16 == 0 && P > 0 && P % 16 == 0 && stride % 4 == 0 && q_at % 4 == 0 && k_at % 4 == 0;
}

extern "C" int axk_lightning_chunked(const float* rows, long stride, int q_at, int k_at, int v_at, const float* decay, float* state,
                                     long state_stride, long copy_elems, const int32_t* chunks, int n_chunks, const int32_t* spans5,
                                     int n_spans, const int32_t* positions, float* y, int heads, int N, int P, float* ends,
                                     long ends_floats, void* stream) {
  const int rc = lightning_sizes_ok("lightning_chunked", heads, N, P, stride, q_at, k_at, v_at, state_stride, copy_elems);
  if (rc != 0) return rc;
  AXK_REQUIRE(axk_lightning_chunked_ok(heads, N, P, stride, q_at, k_at) && ((uintptr_t)rows & 15) == 0 && ((uintptr_t)ends & 15) == 0,
              "lightning_chunked: keys=%d values=%d rows of %ld, or rows are not 16-byte aligned", N, P, stride);
  AXK_REQUIRE(n_spans >= 0 && n_chunks >= n_spans && n_chunks <= 65535 && n_spans <= 65535, "lightning_chunked: %d chunks of %d requests",
              n_chunks, n_spans);
  AXK_REQUIRE(ends != nullptr && ends_floats >= (long)n_chunks * heads * N * P, "lightning_chunked: a workspace of %ld floats", ends_floats);
  if (n_spans == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  lightning_ends_kernel<<<dim3(heads, n_chunks, ceil_div(N, 64)), 256, 0, s>>>(rows, stride, k_at, v_at, decay, chunks, ends, heads, N, P);
  lightning_fold_kernel<<<dim3(n_spans, ceil_div(N * P, 256), heads), 256, 0, s>>>(ends, decay, chunks, spans5, state, state_stride,
                                                                                  copy_elems, positions, heads, N, P);
  lightning_outputs_kernel<<<dim3(heads, n_chunks, ceil_div(P, 16 * LC_VT)), 256, 0, s>>>(rows, stride, q_at, k_at, v_at, decay, chunks,
                                                                                         ends, y, heads, N, P);
  AXK_LAUNCH_CHECK("lightning_chunked");
  return 0;
}
