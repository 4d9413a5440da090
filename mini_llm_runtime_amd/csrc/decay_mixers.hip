// Recurrences with one decay per head and token behind a short causal convolution: the convolution with its
// activation, unit norms and gates; the scan of a matrix state, plain (state spaces) or by the delta rule; and the
// norm of gated heads in equal parts of a row.  All arithmetic is float32; bfloat16 only exists in the activations
// that leave for a matrix product.
#include "api.h"
#include "common.h"

namespace mlr {
namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// ---- convolution, activation, unit norms, gates ----------------------------------------------------------
// p [tokens, width] float32; the channels c of the convolution are its columns column + c.  Per token t of entry e:
//   x[c] = silu(sum_j taps[j, c] * in(t - (n_taps - 1) + j, c) (+ bias[c])),  in() = the entry's inputs in order: this
// step's, before them the n_taps - 1 that row read_rows[e] of `state` [rows, n_taps - 1, channels] carries (oldest
// first; zeros where the entry starts its request).  The entry's last token leaves the newest ones in row write_rows[e].
// The first unit_heads * unit_dim channels are heads, each divided by sqrt(sum of squares + 1e-6); the first
// scaled_heads of them are multiplied by unit_scale.  gates[t, h] = (rate[h] s, w) with s = softplus(p[step_column + h] +
// dt_bias[h]) and w = s, or sigmoid(p[write_column + h]) where write_column >= 0.
// A wavefront per (token, job): a job is one unit head, 256 of the other channels, or the gates of all heads.
constexpr int kPlainChannels = 256;

template <int TAPS>  // 0: any number of taps
__global__ __launch_bounds__(256) void conv_gates_kernel(
    const float* __restrict__ p, int width, int column, const float* __restrict__ taps, const float* __restrict__ bias,
    float* __restrict__ state, const int* __restrict__ read_rows, const int* __restrict__ write_rows,
    const int* __restrict__ token_entry, const int* __restrict__ cu_q, const int* __restrict__ q_starts,
    float* __restrict__ out, float* __restrict__ gates, int channels, int n_taps_any, int unit_heads, int unit_dim,
    int scaled_heads, float unit_scale, const float* __restrict__ rate, const float* __restrict__ dt_bias, int heads,
    int step_column, int write_column, int plain_jobs) {
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x % kWave;
  const int job = blockIdx.y * 4 + threadIdx.x / kWave;
  const int jobs = unit_heads + plain_jobs + 1;
  if (job >= jobs) return;
  const float* row = p + t * width;
  if (job == jobs - 1) {
    for (int h = lane; h < heads; h += kWave) {
      const float s = softplus_f32(row[step_column + h] + dt_bias[h]);
      const float w = write_column >= 0 ? 1.0f / (1.0f + expf(-row[write_column + h])) : s;
      gates[(t * heads + h) * 2] = rate[h] * s;
      gates[(t * heads + h) * 2 + 1] = w;
    }
    return;
  }
  const int n_taps = TAPS > 0 ? TAPS : n_taps_any;
  const int entry = token_entry[t];
  const int first = cu_q[entry];
  const int i = static_cast<int>(t) - first;  // place among the step's tokens of the entry
  const int count = cu_q[entry + 1] - first;
  const int carried = n_taps - 1;
  const bool unit = job < unit_heads;
  const int base = unit ? job * unit_dim : unit_heads * unit_dim + (job - unit_heads) * kPlainChannels;
  const int n = unit ? unit_dim : min(kPlainChannels, channels - base);
  const bool fresh = carried == 0 || q_starts[entry] == 0;
  const float* old = fresh ? nullptr : state + static_cast<int64_t>(read_rows[entry]) * carried * channels;
  auto input = [&](int at, int c) -> float {  // `at` counts from the step's first token of the entry
    if (at >= 0) return p[(static_cast<int64_t>(first) + at) * width + column + c];
    return fresh ? 0.f : old[static_cast<int64_t>(carried + at) * channels + c];
  };
  float v[4];
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int j = lane + u * kWave;
    v[u] = 0.f;
    if (j < n) {
      const int c = base + j;
      float acc = bias != nullptr ? bias[c] : 0.f;
      if constexpr (TAPS > 0) {
        float in[TAPS];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) in[k] = input(i - (TAPS - 1) + k, c);
#pragma unroll
        for (int k = 0; k < TAPS; ++k) acc = fmaf(taps[k * channels + c], in[k], acc);
      } else {
        for (int k = 0; k < n_taps; ++k) acc = fmaf(taps[k * channels + c], input(i - carried + k, c), acc);
      }
      v[u] = silu_f32(acc);
      ss = fmaf(v[u], v[u], ss);
    }
  }
  float factor = 1.0f;
  if (unit) factor = (job < scaled_heads ? unit_scale : 1.0f) / sqrtf(wave_sum(ss) + 1e-6f);
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int j = lane + u * kWave;
    if (j < n) out[t * channels + base + j] = v[u] * factor;
  }
  if (i == count - 1 && carried > 0) {
    float* dst = state + static_cast<int64_t>(write_rows[entry]) * carried * channels;
    for (int s = 0; s < carried; ++s)
      for (int j = lane; j < n; j += kWave)
        dst[static_cast<int64_t>(s) * channels + base + j] = input(count - carried + s, base + j);
  }
}

// ---- the scan, token by token -----------------------------------------------------------------------------
// With (a, w) = gates[t, h], per head:  S <- exp(a) S;  u = w v, or DELTA: u = w (v - S^T k);  S <- S + k u^T;
// o = S^T q (+ skip[h] v).  x [tokens, channels] holds q, k (key_heads * dim each, head h reads key head h / (heads /
// key_heads)) and v (heads * vdim) from columns q_off, k_off, v_off on; the state is row read_rows[entry] of `state`
// [rows, heads, dim, vdim] (zeros where the entry starts its request, whatever the row holds) and goes to row
// write_rows[entry].  A workgroup of four wavefronts owns 64 value columns of one head of one entry: lane (g, c) of a
// wavefront holds a quarter of the rows of column c (consecutive ones: 16-byte LDS reads); eight tokens' q and k at a
// time go through LDS, rows beyond dim as zeros, and the eight after them are on their way from memory meanwhile.
constexpr int kWalkTokens = 8;

template <int R, bool DELTA>  // R: rows of the state a lane holds, dim <= 4 * R
__global__ __launch_bounds__(256) void decay_walk_kernel(
    const float* __restrict__ x, int channels, int q_off, int k_off, int v_off, const float* __restrict__ gates,
    float* __restrict__ state, const int* __restrict__ read_rows, const int* __restrict__ write_rows,
    const int* __restrict__ cu_q, const int* __restrict__ q_starts, const float* __restrict__ skip,
    float* __restrict__ out, int heads, int key_heads, int dim, int vdim) {
  constexpr int MAXD = 4 * R;
  constexpr int kGroup = R + 4;  // floats of a group of rows in LDS: the four groups' 16-byte reads fall into banks of their own
  __shared__ __attribute__((aligned(16))) float sq[kWalkTokens][4][kGroup];
  __shared__ __attribute__((aligned(16))) float sk[kWalkTokens][4][kGroup];
  __shared__ float sv[kWalkTokens][64];
  __shared__ float sg[kWalkTokens][2];
  const int entry = blockIdx.x;
  const int h = blockIdx.y;
  const int kh = h / (heads / key_heads);
  const int tid = threadIdx.x;
  const int lane = tid % kWave;
  const int wave = tid / kWave;
  const int g = lane / 16;  // this lane's rows: g * R .. g * R + R - 1
  const int c_local = wave * 16 + lane % 16;
  const int col = blockIdx.z * 64 + c_local;
  const bool col_ok = col < vdim;
  const int t_begin = cu_q[entry];
  const int t_end = cu_q[entry + 1];
  const bool fresh = q_starts[entry] == 0;
  const int64_t per_head = static_cast<int64_t>(dim) * vdim;
  const float* src = state + (static_cast<int64_t>(read_rows[entry]) * heads + h) * per_head;
  float* dst = state + (static_cast<int64_t>(write_rows[entry]) * heads + h) * per_head;

  constexpr int kPer = kWalkTokens * MAXD / 256;
  float rq[kPer], rk[kPer], rv[2], rg[2];
  auto fetch = [&](int t0) {
    const int nb = min(kWalkTokens, t_end - t0);
#pragma unroll
    for (int u = 0; u < kPer; ++u) {
      const int idx = tid + u * 256;
      const int tt = idx / MAXD;
      const int r = idx - tt * MAXD;
      const bool in = tt < nb && r < dim;
      const float* row = x + static_cast<int64_t>(t0 + (in ? tt : 0)) * channels + kh * dim + (in ? r : 0);
      rq[u] = in ? row[q_off] : 0.f;
      rk[u] = in ? row[k_off] : 0.f;
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int idx = tid + u * 256;
      const int tt = idx / 64;
      const int c = blockIdx.z * 64 + (idx - tt * 64);
      const bool in = tt < nb && c < vdim;
      rv[u] = in ? x[static_cast<int64_t>(t0 + tt) * channels + v_off + h * vdim + c] : 0.f;
    }
    rg[0] = rg[1] = 0.f;
    if (tid < nb) {
      rg[0] = gates[(static_cast<int64_t>(t0 + tid) * heads + h) * 2];
      rg[1] = gates[(static_cast<int64_t>(t0 + tid) * heads + h) * 2 + 1];
    }
  };
  auto stash = [&]() {
#pragma unroll
    for (int u = 0; u < kPer; ++u) {
      const int idx = tid + u * 256;
      const int tt = idx / MAXD;
      const int r = idx - tt * MAXD;
      sq[tt][r / R][r % R] = rq[u];
      sk[tt][r / R][r % R] = rk[u];
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int idx = tid + u * 256;
      sv[idx / 64][idx % 64] = rv[u];
    }
    if (tid < kWalkTokens) {
      sg[tid][0] = expf(rg[0]);
      sg[tid][1] = rg[1];
    }
  };
  fetch(t_begin);
  float S[R];
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int r = g * R + j;
    S[j] = (r < dim && !fresh && col_ok) ? src[static_cast<int64_t>(r) * vdim + col] : 0.f;
  }
  const float d_skip = skip != nullptr ? skip[h] : 0.f;

  for (int t0 = t_begin; t0 < t_end; t0 += kWalkTokens) {
    const int nb = min(kWalkTokens, t_end - t0);
    __syncthreads();  // the tokens before are walked
    stash();
    __syncthreads();
    if (t0 + kWalkTokens < t_end) fetch(t0 + kWalkTokens);  // on their way during the walk
    for (int tt = 0; tt < nb; ++tt) {
      const float keep = sg[tt][0];
      const float w = sg[tt][1];
      const float v = sv[tt][c_local];
      float u = v;
      if constexpr (DELTA) {
        float held = 0.f;
#pragma unroll
        for (int j = 0; j < R; j += 4) {
          const f32x4 k4 = *reinterpret_cast<const f32x4*>(&sk[tt][g][j]);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[j + e] *= keep;
            held = fmaf(S[j + e], k4[e], held);
          }
        }
        held += __shfl_xor(held, 16, kWave);
        held += __shfl_xor(held, 32, kWave);
        u = v - held;
      }
      u *= w;
      float o = 0.f;
#pragma unroll
      for (int j = 0; j < R; j += 4) {
        const f32x4 k4 = *reinterpret_cast<const f32x4*>(&sk[tt][g][j]);
        const f32x4 q4 = *reinterpret_cast<const f32x4*>(&sq[tt][g][j]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[j + e] = DELTA ? fmaf(k4[e], u, S[j + e]) : fmaf(keep, S[j + e], k4[e] * u);
          o = fmaf(S[j + e], q4[e], o);
        }
      }
      o += __shfl_xor(o, 16, kWave);
      o += __shfl_xor(o, 32, kWave);
      if (g == 0 && col_ok)
        out[(static_cast<int64_t>(t0 + tt) * heads + h) * vdim + col] = fmaf(d_skip, v, o);
    }
  }
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int r = g * R + j;
    if (r < dim && col_ok) dst[static_cast<int64_t>(r) * vdim + col] = S[j];
  }
}

// ---- one token per entry: convolution, gates and scan in one kernel ---------------------------------------------
// What conv_gates_kernel and decay_walk_kernel do for a step in which every entry has a single token (entry e is token
// e), for convolutions of up to kStepTaps taps.  A workgroup owns 64 value columns of one head of one entry and makes
// the head's q and k and its columns' v itself; the carried inputs of q's and k's channels are written by the first
// head of those that share them (and its first columns), those of v's channels by their owner.
constexpr int kStepTaps = 4;

struct StepConv {
  const float* p;  // [tokens, width]; the convolution's channels start at `column`
  int width, column, n_taps;
  const float *taps, *bias;
  float* carried;  // [rows, n_taps - 1, channels]
  const int *read_rows, *write_rows;
  const float *rate, *dt_bias;
  int step_column, write_column;
  float unit_scale;  // of q (unit heads only)
};

template <int R, bool DELTA>  // R: rows of the state a lane holds, dim <= 4 * R; DELTA: unit q and k, else as they are
__global__ __launch_bounds__(256) void decay_step_kernel(StepConv in, int channels, int q_off, int k_off, int v_off,
                                                         float* __restrict__ state, const int* __restrict__ read_rows,
                                                         const int* __restrict__ write_rows,
                                                         const int* __restrict__ q_starts, const float* __restrict__ skip,
                                                         float* __restrict__ out, int heads, int key_heads, int dim,
                                                         int vdim) {
  constexpr int MAXD = 4 * R;
  constexpr int kGroup = R + 4;
  constexpr int kRounds = (2 * MAXD + 255) / 256;
  __shared__ __attribute__((aligned(16))) float qk[2][4][kGroup];
  __shared__ float sv[64];
  __shared__ float sg[2];
  __shared__ float squares[kRounds][4];
  const int entry = blockIdx.x;
  const int h = blockIdx.y;
  const int group = heads / key_heads;
  const int kh = h / group;
  const int tid = threadIdx.x;
  const int lane = tid % kWave;
  const int wave = tid / kWave;
  const int g = lane / 16;
  const int c_local = wave * 16 + lane % 16;
  const int col = blockIdx.z * 64 + c_local;
  const bool col_ok = col < vdim;
  const bool fresh = q_starts[entry] == 0;
  const int64_t per_head = static_cast<int64_t>(dim) * vdim;
  const float* src = state + (static_cast<int64_t>(read_rows[entry]) * heads + h) * per_head;
  float* dst = state + (static_cast<int64_t>(write_rows[entry]) * heads + h) * per_head;
  // the state is on its way while the token's q, k and v are made (what is absent reads element 0)
  float S[R];
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int r = g * R + j;
    S[j] = src[(r < dim && col_ok) ? static_cast<int64_t>(r) * vdim + col : 0];
  }
  const float* row = in.p + static_cast<int64_t>(entry) * in.width;
  const int carried = in.n_taps - 1;
  const bool keeps = carried > 0;
  const float* old = keeps ? in.carried + static_cast<int64_t>(in.read_rows[entry]) * carried * channels : row;
  float* kept = keeps ? in.carried + static_cast<int64_t>(in.write_rows[entry]) * carried * channels : nullptr;
  auto convolved = [&](int c, bool owner) {  // channel c: convolution and activation; `owner` writes its inputs
    float x[kStepTaps], w[kStepTaps];
    const float now = row[in.column + c];
#pragma unroll
    for (int k = 0; k < kStepTaps - 1; ++k)  // x[k]: the input k + 1 tokens ago
      x[k] = k < carried && !fresh ? old[static_cast<int64_t>(carried - 1 - k) * channels + c] : 0.f;
#pragma unroll
    for (int k = 0; k < kStepTaps; ++k) w[k] = k <= carried ? in.taps[static_cast<int64_t>(carried - k) * channels + c] : 0.f;
    float acc = in.bias != nullptr ? in.bias[c] : 0.f;
#pragma unroll
    for (int k = kStepTaps - 1; k > 0; --k)
      if (k <= carried) acc = fmaf(w[k], x[k - 1], acc);  // the oldest first, as in conv_gates_kernel
    acc = fmaf(w[0], now, acc);
    if (owner && keeps) {
#pragma unroll
      for (int k = 0; k < kStepTaps - 1; ++k)
        if (k < carried) kept[static_cast<int64_t>(carried - 1 - k) * channels + c] = k == 0 ? now : x[k - 1];
    }
    return silu_f32(acc);
  };
  const bool first = h == kh * group && blockIdx.z == 0;
  float made[kRounds];
#pragma unroll
  for (int u = 0; u < kRounds; ++u) {
    const int idx = tid + u * 256;
    const int which = idx / MAXD;  // 0: q, 1: k
    const int r = idx % MAXD;
    made[u] = 0.f;
    if (which < 2 && r < dim) made[u] = convolved((which ? k_off : q_off) + kh * dim + r, first);
    if constexpr (DELTA) {
      const float ss = wave_sum(made[u] * made[u]);
      if (lane == 0) squares[u][wave] = ss;
    }
  }
  if (wave == 3) {
    const int c = blockIdx.z * 64 + lane;
    sv[lane] = c < vdim ? convolved(v_off + h * vdim + c, true) : 0.f;
  }
  if (tid == 128) {
    const float s = softplus_f32(row[in.step_column + h] + in.dt_bias[h]);
    sg[0] = expf(in.rate[h] * s);
    sg[1] = in.write_column >= 0 ? 1.0f / (1.0f + expf(-row[in.write_column + h])) : s;
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < kRounds; ++u) {
    const int idx = tid + u * 256;
    const int which = idx / MAXD;
    const int r = idx % MAXD;
    if (which < 2) {
      float v = made[u];
      if constexpr (DELTA) {
        float ss = 0.f;
#pragma unroll
        for (int a = 0; a < kRounds; ++a)
#pragma unroll
          for (int b = 0; b < 4; ++b)
            if ((a * 256 + b * 64) / MAXD == which) ss += squares[a][b];
        v *= (which ? 1.0f : in.unit_scale) / sqrtf(ss + 1e-6f);
      }
      qk[which][r / R][r % R] = v;
    }
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < R; ++j)
    if (!(g * R + j < dim && col_ok) || fresh) S[j] = 0.f;
  const float keep = sg[0];
  const float v = sv[c_local];
  float u = v;
  if constexpr (DELTA) {
    float held = 0.f;
#pragma unroll
    for (int j = 0; j < R; j += 4) {
      const f32x4 k4 = *reinterpret_cast<const f32x4*>(&qk[1][g][j]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[j + e] *= keep;
        held = fmaf(S[j + e], k4[e], held);
      }
    }
    held += __shfl_xor(held, 16, kWave);
    held += __shfl_xor(held, 32, kWave);
    u = v - held;
  }
  u *= sg[1];
  float o = 0.f;
#pragma unroll
  for (int j = 0; j < R; j += 4) {
    const f32x4 k4 = *reinterpret_cast<const f32x4*>(&qk[1][g][j]);
    const f32x4 q4 = *reinterpret_cast<const f32x4*>(&qk[0][g][j]);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      S[j + e] = DELTA ? fmaf(k4[e], u, S[j + e]) : fmaf(keep, S[j + e], k4[e] * u);
      o = fmaf(S[j + e], q4[e], o);
    }
  }
  o += __shfl_xor(o, 16, kWave);
  o += __shfl_xor(o, 32, kWave);
  if (g == 0 && col_ok)
    out[(static_cast<int64_t>(entry) * heads + h) * vdim + col] = fmaf(skip != nullptr ? skip[h] : 0.f, v, o);
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int r = g * R + j;
    if (r < dim && col_ok) dst[static_cast<int64_t>(r) * vdim + col] = S[j];
  }
}

// ---- the scan, 64 tokens at a time on the matrix cores ----------------------------------------------------------
// In true 32-bit: v_mfma_f32_16x16x4_f32 takes and sums float32.  Within a chunk of n tokens (local index i, j; what is
// beyond n is zero) with S the state before it, A_i = a_0 + .. + a_i (summed in float64: only differences of it are
// used, and they may be small beside it) and e(i, j) = exp(A_i - A_j):
//     DELTA: u solves u_i + sum_{j<i} w_i e(i, j) (k_i . k_j) u_j = w_i v_i - w_i exp(A_i) S^T k_i, i.e. with L the strictly
//     lower triangular matrix of the sum, U = U0 - X S for (I + L) [X | U0] = [w exp(A) K | w V];    else u_i = w_i v_i;
//     o_i = exp(A_i) S^T q_i + sum_{j<=i} e(i, j) (q_i . k_j) u_j,     S' = exp(A_n) S + sum_j e(n, j) k_j u_j^T.
// decay_local_kernel, all chunks of all entries at once: the parts that do not need S (DELTA: X and U0 by block forward
// substitution; else the chunk's share of S').  The walk over an entry's chunks: delta_carry_kernel (two products a
// chunk) or plain_carry_kernel (element by element); both leave the state BEFORE every chunk.  decay_apply_kernel, all chunks at
// once again, makes the outputs.
// Lane layouts of the product D[16x16] += A[16x4] B[4x16]: lane l holds A[l % 16][l / 16], B[l / 16][l % 16] and
// D[4 (l / 16) + e][l % 16], e = 0..3.  A sum over 16 values of k is four such products, and any order of k will do if
// both operands keep it: product e takes k = 4 (l / 16) + e.  So operands are read as four consecutive k (16 bytes) a
// lane, and a D tile is, register by register, the B operand of the next product over its rows.
constexpr int kChunk = 64;
constexpr int kMatLd = kChunk + 8;  // row of a 64 x 64 matrix in LDS: 32 bytes modulo 64 keeps 16-byte reads of 16 rows off each other's banks

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

__host__ __device__ __forceinline__ int chunks_of(int tokens) { return (tokens + kChunk - 1) / kChunk; }

// Which entry chunk number `chunk` (counted through the entries in order) belongs to, its first token and its tokens.
__device__ inline bool find_chunk(const int* __restrict__ cu_q, int entries, int chunk, int& entry, int& place, int& t0, int& n) {
  for (int e = 0; e < entries; ++e) {
    const int have = chunks_of(cu_q[e + 1] - cu_q[e]);
    if (chunk < have) {
      entry = e;
      place = chunk;
      t0 = cu_q[e] + chunk * kChunk;
      n = min(kChunk, cu_q[e + 1] - t0);
      return true;
    }
    chunk -= have;
  }
  return false;
}

// The chunk's A_i (float64) and w_i into LDS, by the first wavefront.
__device__ __forceinline__ void chunk_gates(const float* __restrict__ gates, int heads, int h, int t0, int n, double* As, float* ws) {
  if (threadIdx.x < kChunk) {
    const int i = threadIdx.x;
    const float* g = gates + (static_cast<int64_t>(t0 + min(i, n - 1)) * heads + h) * 2;
    double a = i < n ? static_cast<double>(g[0]) : 0.0;
#pragma unroll
    for (int d = 1; d < kChunk; d *= 2) {
      const double before = __shfl_up(a, d, kWave);
      if (i >= d) a += before;
    }
    As[i] = a;
    ws[i] = i < n ? g[1] : 0.f;
  }
}

// Rows of one head of the chunk (columns `at` .. of x), zero beyond n and dim, into LDS rows of LD floats.
template <int DP, int LD>
__device__ __forceinline__ void chunk_rows(const float* __restrict__ x, int channels, int at, int t0, int n, int dim, float* rows) {
  constexpr int kEach = kChunk * DP / 256;
  float v[kEach];
#pragma unroll
  for (int u = 0; u < kEach; ++u) {
    const int idx = threadIdx.x + u * 256;
    const int i = idx / DP, d = idx % DP;
    v[u] = x[static_cast<int64_t>(t0 + min(i, n - 1)) * channels + at + min(d, dim - 1)];
  }
#pragma unroll
  for (int u = 0; u < kEach; ++u) {
    const int idx = threadIdx.x + u * 256;
    const int i = idx / DP, d = idx % DP;
    rows[i * LD + d] = (i < n && d < dim) ? v[u] : 0.f;
  }
}

// The lower triangle of 4 x 4 blocks of 16 x 16, diagonal included, as a list: block b is (row, column).
__device__ __forceinline__ void triangle_block(int b, int& row, int& column) {
  row = b < 1 ? 0 : b < 3 ? 1 : b < 6 ? 2 : 3;
  column = b - row * (row + 1) / 2;
}

// rows a[16 bi ..] times rows b[16 bj ..] transposed, both [64][LD] in LDS: a D tile.
template <int DP, int LD>
__device__ __forceinline__ f32x4 rows_product(const float* a, const float* b, int bi, int bj, int r16, int quad) {
  f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
  for (int g = 0; g < DP / 16; ++g) {
    const f32x4 av = *reinterpret_cast<const f32x4*>(&a[(16 * bi + r16) * LD + 16 * g + 4 * quad]);
    const f32x4 bv = *reinterpret_cast<const f32x4*>(&b[(16 * bj + r16) * LD + 16 * g + 4 * quad]);
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[e % 2] = mfma_f32(av[e], bv[e], acc[e % 2]);
  }
  return acc[0] + acc[1];
}

// Where a scan's scratch memory holds what, per chunk and head (offsets in floats): the state before the chunk [DP, vpad]; for
// the delta rule X [64, DP], K [64, DP] (zero padded), U [64, vpad] (U0, then U) and e(n, j) [64]; exp(A_n).
struct ChunkScratch {
  float *state, *x, *k, *u, *last, *decay;
  int dp, vpad;
};
__host__ __device__ inline int64_t scratch_floats_per_chunk(int dp, int vpad, int delta) {
  return static_cast<int64_t>(dp) * vpad + (delta ? 2 * kChunk * dp + kChunk * vpad + kChunk : 0) + 1;
}
inline ChunkScratch chunk_scratch(float* base, int64_t cells, int dp, int vpad, int delta) {
  ChunkScratch s;
  s.dp = dp;
  s.vpad = vpad;
  s.state = base;
  float* at = base + cells * dp * vpad;
  s.x = at;
  if (delta) at += cells * kChunk * dp;
  s.k = at;
  if (delta) at += cells * kChunk * dp;
  s.u = at;
  if (delta) at += cells * kChunk * vpad;
  s.last = at;
  if (delta) at += cells * kChunk;
  s.decay = at;
  return s;
}

template <int DP, bool DELTA>
__global__ __launch_bounds__(256) void decay_local_kernel(const float* __restrict__ x, int channels, int k_off, int v_off,
                                                          const float* __restrict__ gates, const int* __restrict__ cu_q,
                                                          int entries, int heads, int key_heads, int dim, int vdim,
                                                          ChunkScratch out) {
  constexpr int LD = DELTA ? DP + 8 : DP + 4;  // DELTA reads four k of a row at a time, else single elements of rows 4 apart
  __shared__ __attribute__((aligned(16))) float Ks[kChunk * LD];
  __shared__ __attribute__((aligned(16))) float Ls[DELTA ? kChunk * kMatLd : 4];      // -L
  __shared__ __attribute__((aligned(16))) float Ti[DELTA ? 4 * 16 * 24 : 4];         // inverses of I + L's diagonal blocks
  __shared__ double As[kChunk];
  __shared__ float ws[kChunk];
  int entry, place, t0, n;
  if (!find_chunk(cu_q, entries, blockIdx.x, entry, place, t0, n)) return;  // the grid is sized for the most chunks
  const int h = blockIdx.y;
  const int kh = h / (heads / key_heads);
  const int tid = threadIdx.x;
  const int lane = tid % kWave;
  const int w = __builtin_amdgcn_readfirstlane(tid / kWave);
  const int r16 = lane % 16;
  const int quad = lane / 16;
  const int64_t cell = static_cast<int64_t>(blockIdx.x) * heads + h;
  const int vpad = out.vpad;
  chunk_gates(gates, heads, h, t0, n, As, ws);
  chunk_rows<DP, LD>(x, channels, k_off + kh * dim, t0, n, dim, Ks);
  __syncthreads();
  const double a_last = As[kChunk - 1];
  if (tid == 0) out.decay[cell] = expf(static_cast<float>(a_last));

  // values of a strip of 16 columns, rows 16 b + 4 quad + e
  auto values = [&](int strip, f32x4 (&v)[4]) {
    const int c = strip * 16 + r16;
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int row = 16 * b + 4 * quad + e;
        v[b][e] = x[static_cast<int64_t>(t0 + min(row, n - 1)) * channels + v_off + static_cast<int64_t>(h) * vdim + min(c, vdim - 1)];
      }
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (!(16 * b + 4 * quad + e < n && c < vdim)) v[b][e] = 0.f;
  };

  if constexpr (DELTA) {
    if (tid < kChunk) out.last[cell * kChunk + tid] = expf(static_cast<float>(a_last - As[tid]));
    for (int b = w; b < 10; b += 4) {
      int bi, bj;
      triangle_block(b, bi, bj);
      const f32x4 dot = rows_product<DP, LD>(Ks, Ks, bi, bj, r16, quad);
      const int j = 16 * bj + r16;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 16 * bi + 4 * quad + e;
        Ls[i * kMatLd + j] = j < i ? -ws[i] * expf(static_cast<float>(As[i] - As[j])) * dot[e] : 0.f;
      }
    }
    // K as the carry kernel reads it
    for (int idx = tid; idx < kChunk * DP; idx += 256) out.k[cell * kChunk * DP + idx] = Ks[idx / DP * LD + idx % DP];
    __syncthreads();
    {
      // column r16 of the inverse of diagonal block w, by forward substitution (every 16 lanes the same)
      float t[16];
      const float* block = &Ls[16 * w * kMatLd + 16 * w];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float acc = i == r16 ? 1.0f : 0.f;
#pragma unroll
        for (int j = 0; j < i; ++j) acc = fmaf(block[i * kMatLd + j], t[j], acc);
        t[i] = acc;
      }
      if (quad == 0)
#pragma unroll
        for (int i = 0; i < 16; ++i) Ti[(16 * w + i) * 24 + r16] = t[i];
    }
    __syncthreads();
    const int strips = DP / 16 + vpad / 16;
    for (int s = w; s < strips; s += 4) {
      f32x4 r[4];
      if (s < DP / 16) {
#pragma unroll
        for (int b = 0; b < 4; ++b)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int row = 16 * b + 4 * quad + e;
            r[b][e] = ws[row] * expf(static_cast<float>(As[row])) * Ks[row * LD + 16 * s + r16];
          }
      } else {
        values(s - DP / 16, r);
#pragma unroll
        for (int b = 0; b < 4; ++b)
#pragma unroll
          for (int e = 0; e < 4; ++e) r[b][e] *= ws[16 * b + 4 * quad + e];
      }
      f32x4 solved[4];
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        f32x4 acc = r[b];
#pragma unroll
        for (int k = 0; k < b; ++k) {
          const f32x4 l = *reinterpret_cast<const f32x4*>(&Ls[(16 * b + r16) * kMatLd + 16 * k + 4 * quad]);
#pragma unroll
          for (int e = 0; e < 4; ++e) acc = mfma_f32(l[e], solved[k][e], acc);
        }
        const f32x4 t = *reinterpret_cast<const f32x4*>(&Ti[(16 * b + r16) * 24 + 4 * quad]);
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) y = mfma_f32(t[e], acc[e], y);
        solved[b] = y;
      }
      float* dst = s < DP / 16 ? out.x + cell * kChunk * DP + 16 * s : out.u + cell * kChunk * vpad + 16 * (s - DP / 16);
      const int stride = s < DP / 16 ? DP : vpad;
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) dst[static_cast<int64_t>(16 * b + 4 * quad + e) * stride + r16] = solved[b][e];
    }
  } else {
    float factor[16];
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int row = 16 * b + 4 * quad + e;
        factor[4 * b + e] = ws[row] * expf(static_cast<float>(a_last - As[row]));
      }
    for (int s = w; s < vpad / 16; s += 4) {
      f32x4 v[4];
      values(s, v);
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) v[b][e] *= factor[4 * b + e];
      float* dst = out.state + cell * DP * vpad + 16 * s + r16;
#pragma unroll
      for (int dt = 0; dt < DP / 16; ++dt) {
        f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int b = 0; b < 4; ++b)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            acc[e % 2] = mfma_f32(Ks[(16 * b + 4 * quad + e) * LD + 16 * dt + r16], v[b][e], acc[e % 2]);
#pragma unroll
        for (int e = 0; e < 4; ++e) dst[static_cast<int64_t>(16 * dt + 4 * quad + e) * vpad] = acc[0][e] + acc[1][e];
      }
    }
  }
}

// S' = exp(A_n) S + (the chunk's share), element by element; leaves the state before every chunk where its share was.
__global__ __launch_bounds__(256) void plain_carry_kernel(float* __restrict__ state, const int* __restrict__ read_rows,
                                                          const int* __restrict__ write_rows, const int* __restrict__ cu_q,
                                                          const int* __restrict__ q_starts, int heads, int dim, int vdim,
                                                          ChunkScratch s) {
  const int entry = blockIdx.x;
  const int h = blockIdx.y;
  const int idx = blockIdx.z * 256 + threadIdx.x;
  if (idx >= s.dp * s.vpad) return;
  const int d = idx / s.vpad;
  const int v = idx - d * s.vpad;
  const bool real = d < dim && v < vdim;
  const int count = chunks_of(cu_q[entry + 1] - cu_q[entry]);
  int first = 0;
  for (int e = 0; e < entry; ++e) first += chunks_of(cu_q[e + 1] - cu_q[e]);
  const int64_t head_state = static_cast<int64_t>(dim) * vdim;
  float value = 0.f;
  if (real && q_starts[entry] > 0)
    value = state[(static_cast<int64_t>(read_rows[entry]) * heads + h) * head_state + static_cast<int64_t>(d) * vdim + v];
  const int64_t cells = static_cast<int64_t>(s.dp) * s.vpad;
  float* at = s.state + (static_cast<int64_t>(first) * heads + h) * cells + idx;
  const float* decay = s.decay + static_cast<int64_t>(first) * heads + h;
  for (int c0 = 0; c0 < count; c0 += 8) {  // eight chunks' loads on their way at a time
    float add[8], keep[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const int64_t c = min(c0 + k, count - 1);
      add[k] = at[c * heads * cells];
      keep[k] = decay[c * heads];
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      if (c0 + k < count) {
        at[static_cast<int64_t>(c0 + k) * heads * cells] = value;
        value = fmaf(keep[k], value, add[k]);
      }
    }
  }
  if (real)
    state[(static_cast<int64_t>(write_rows[entry]) * heads + h) * head_state + static_cast<int64_t>(d) * vdim + v] = value;
}

// The delta rule's walk over an entry's chunks for 16 value columns of one head: U = U0 - X S, S' = exp(A_n) S + K^T (e(n, .) U).
// Wavefront w owns the rows 16 w .. of U and every fourth 16-row tile of S (in registers, a D tile each); both go
// through LDS as B operands.  A chunk's X, K and U0 are asked for a whole chunk ahead.  All strips of a head read the
// same X and K: workgroup b runs on accelerator die b % 8, so a head's strips are dealt to one die and share its L2.
template <int DP>
struct CarryOperands {
  f32x4 x[DP / 16], u0, last;
  float k[(DP / 16 + 3) / 4][16];
  float keep;
};

constexpr int kDies = 8;

template <int DP>
__global__ __launch_bounds__(256) void delta_carry_kernel(float* __restrict__ state, const int* __restrict__ read_rows,
                                                          const int* __restrict__ write_rows, const int* __restrict__ cu_q,
                                                          const int* __restrict__ q_starts, int entries, int heads, int dim,
                                                          int vdim, ChunkScratch s) {
  constexpr int kTiles = DP / 16;
  constexpr int kOwn = (kTiles + 3) / 4;  // tiles of S a wavefront owns at most
  __shared__ __attribute__((aligned(16))) f32x4 Sb[kTiles][kWave];
  __shared__ __attribute__((aligned(16))) f32x4 Ub[4][kWave];
  const int vpad = s.vpad;
  const int strips = vpad / 16;
  const int slot = blockIdx.x / kDies;
  const int unit = slot / strips * kDies + blockIdx.x % kDies;  // (entry, head)
  const int strip = slot % strips;
  if (unit >= entries * heads) return;
  const int entry = unit / heads;
  const int h = unit - entry * heads;
  const int tid = threadIdx.x;
  const int lane = tid % kWave;
  const int w = __builtin_amdgcn_readfirstlane(tid / kWave);
  const int r16 = lane % 16;
  const int quad = lane / 16;
  const int col = strip * 16 + r16;
  const int count = chunks_of(cu_q[entry + 1] - cu_q[entry]);
  int first = 0;
  for (int e = 0; e < entry; ++e) first += chunks_of(cu_q[e + 1] - cu_q[e]);
  const int64_t head_state = static_cast<int64_t>(dim) * vdim;

  f32x4 S[kOwn];
  const bool fresh = q_starts[entry] == 0;
  const float* src = state + (static_cast<int64_t>(read_rows[entry]) * heads + h) * head_state;
#pragma unroll
  for (int o = 0; o < kOwn; ++o)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * (w + 4 * o) + 4 * quad + e;
      S[o][e] = (!fresh && d < dim && col < vdim) ? src[static_cast<int64_t>(d) * vdim + col] : 0.f;
    }

  auto fetch = [&](CarryOperands<DP>& op, int c) {
    const int64_t cell = static_cast<int64_t>(first + c) * heads + h;
    const float* xr = s.x + (cell * kChunk + 16 * w + r16) * DP + 4 * quad;
#pragma unroll
    for (int g = 0; g < kTiles; ++g) op.x[g] = *reinterpret_cast<const f32x4*>(xr + 16 * g);
    const float* ur = s.u + (cell * kChunk + 16 * w + 4 * quad) * vpad + col;
#pragma unroll
    for (int e = 0; e < 4; ++e) op.u0[e] = ur[e * vpad];
    op.last = *reinterpret_cast<const f32x4*>(s.last + cell * kChunk + 16 * w + 4 * quad);
    op.keep = s.decay[cell];
    const float* kr = s.k + (cell * kChunk + 4 * quad) * DP + r16;
#pragma unroll
    for (int o = 0; o < kOwn; ++o) {
      const int tile = min(w + 4 * o, kTiles - 1);
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) op.k[o][4 * b + e] = kr[(16 * b + e) * DP + 16 * tile];
    }
  };
  auto step = [&](const CarryOperands<DP>& op, CarryOperands<DP>& next, int c) {
    const int64_t cell = static_cast<int64_t>(first + c) * heads + h;
    float* before = s.state + cell * DP * vpad + col;
#pragma unroll
    for (int o = 0; o < kOwn; ++o) {
      const int tile = w + 4 * o;
      if (kTiles % 4 == 0 || tile < kTiles) Sb[tile][lane] = S[o];
    }
    __syncthreads();
    // asked for without a condition (past the end: the last chunk again): a load inside a conditional block would make the
    // compiler wait for every load on its way where the block ends
    fetch(next, min(c + 1, count - 1));
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int o = 0; o < kOwn; ++o) {
      const int tile = w + 4 * o;
      if (kTiles % 4 == 0 || tile < kTiles)
#pragma unroll
        for (int e = 0; e < 4; ++e) before[static_cast<int64_t>(16 * tile + 4 * quad + e) * vpad] = S[o][e];
    }
    f32x4 held[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int g = 0; g < kTiles; ++g) {
      const f32x4 sb = Sb[g][lane];
#pragma unroll
      for (int e = 0; e < 4; ++e) held[e % 2] = mfma_f32(op.x[g][e], sb[e], held[e % 2]);
    }
    const f32x4 u = op.u0 - (held[0] + held[1]);
    Ub[w][lane] = u * op.last;
    __syncthreads();
    float* ur = s.u + (cell * kChunk + 16 * w + 4 * quad) * vpad + col;
#pragma unroll
    for (int e = 0; e < 4; ++e) ur[e * vpad] = u[e];
    f32x4 ub[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) ub[b] = Ub[b][lane];
#pragma unroll
    for (int o = 0; o < kOwn; ++o) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      S[o] *= op.keep;
#pragma unroll
      for (int b = 0; b < 4; ++b) {
#pragma unroll
        for (int e = 0; e < 4; e += 2) {
          S[o] = mfma_f32(op.k[o][4 * b + e], ub[b][e], S[o]);
          acc = mfma_f32(op.k[o][4 * b + e + 1], ub[b][e + 1], acc);
        }
      }
      S[o] += acc;
    }
  };
  CarryOperands<DP> even, odd;
  fetch(even, 0);
  for (int c = 0; c < count; c += 2) {
    step(even, odd, c);
    if (c + 1 < count) step(odd, even, c + 1);
  }
  float* dst = state + (static_cast<int64_t>(write_rows[entry]) * heads + h) * head_state;
#pragma unroll
  for (int o = 0; o < kOwn; ++o)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * (w + 4 * o) + 4 * quad + e;
      if (d < dim && col < vdim) dst[static_cast<int64_t>(d) * vdim + col] = S[o][e];
    }
}

// The outputs of a chunk: o_i = exp(A_i) S^T q_i + sum_{j<=i} e(i, j) (q_i . k_j) u_j (+ skip v_i).  The scores take the
// place of the keys in LDS; a wavefront then owns every fourth strip of 16 value columns, whose state and u it
// reads once for all 64 rows.
template <int DP, bool DELTA>
__global__ __launch_bounds__(256) void decay_apply_kernel(const float* __restrict__ x, int channels, int q_off, int k_off,
                                                          int v_off, const float* __restrict__ gates,
                                                          const int* __restrict__ cu_q, const int* __restrict__ q_starts,
                                                          const float* __restrict__ skip, float* __restrict__ out,
                                                          int entries, int heads, int key_heads, int dim, int vdim,
                                                          ChunkScratch s) {
  constexpr int LD = DP + 8;
  extern __shared__ __attribute__((aligned(16))) float apply_lds[];
  float* const Qs = apply_lds;            // [64][LD]
  float* const Ks = Qs + kChunk * LD;     // [64][LD], then the scores [64][kMatLd]
  float* const Ps = Ks;
  __shared__ double As[kChunk];
  __shared__ float ws[kChunk];
  int entry, place, t0, n;
  if (!find_chunk(cu_q, entries, blockIdx.x, entry, place, t0, n)) return;
  const int h = blockIdx.y;
  const int kh = h / (heads / key_heads);
  const int tid = threadIdx.x;
  const int lane = tid % kWave;
  const int w = __builtin_amdgcn_readfirstlane(tid / kWave);
  const int r16 = lane % 16;
  const int quad = lane / 16;
  const int64_t cell = static_cast<int64_t>(blockIdx.x) * heads + h;
  const int vpad = s.vpad;
  chunk_gates(gates, heads, h, t0, n, As, ws);
  chunk_rows<DP, LD>(x, channels, q_off + kh * dim, t0, n, dim, Qs);
  chunk_rows<DP, LD>(x, channels, k_off + kh * dim, t0, n, dim, Ks);
  __syncthreads();
  f32x4 dots[3];
#pragma unroll
  for (int u = 0; u < 3; ++u) {
    const int b = w + 4 * u;
    if (b < 10) {
      int bi, bj;
      triangle_block(b, bi, bj);
      dots[u] = rows_product<DP, LD>(Qs, Ks, bi, bj, r16, quad);
    }
  }
  __syncthreads();  // the keys are done with
#pragma unroll
  for (int u = 0; u < 3; ++u) {
    const int b = w + 4 * u;
    if (b < 10) {
      int bi, bj;
      triangle_block(b, bi, bj);
      const int j = 16 * bj + r16;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 16 * bi + 4 * quad + e;
        Ps[i * kMatLd + j] = j <= i ? expf(static_cast<float>(As[i] - As[j])) * (DELTA ? 1.0f : ws[j]) * dots[u][e] : 0.f;
      }
    }
  }
  __syncthreads();
  const bool carried = !(place == 0 && q_starts[entry] == 0);  // else the state before the chunk is zero
  const float d_skip = skip != nullptr ? skip[h] : 0.f;
  // a strip's u and state, all asked for before the first is used
  struct Strip {
    f32x4 u[4], s[DP / 16];
  };
  auto fetch = [&](Strip& t, int strip) {
    const int c = strip * 16 + r16;
    if constexpr (DELTA) {
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) t.u[b][e] = s.u[(cell * kChunk + 16 * b + 4 * quad + e) * vpad + c];
    } else {
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          t.u[b][e] = x[static_cast<int64_t>(t0 + min(16 * b + 4 * quad + e, n - 1)) * channels + v_off +
                        static_cast<int64_t>(h) * vdim + min(c, vdim - 1)];
    }
    const float* before = s.state + cell * DP * vpad + c;  // zeros before a request's first chunk
#pragma unroll
    for (int g = 0; g < DP / 16; ++g)
#pragma unroll
      for (int e = 0; e < 4; ++e) t.s[g][e] = before[static_cast<int64_t>(16 * g + 4 * quad + e) * vpad];
    __builtin_amdgcn_sched_barrier(0);  // all asked for here, not each where it is used
  };
  auto compute = [&](const Strip& t, int strip) {
    const int c = strip * 16 + r16;
    f32x4 o[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) o[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (carried) {
#pragma unroll
      for (int g = 0; g < DP / 16; ++g) {
        f32x4 q[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) q[b] = *reinterpret_cast<const f32x4*>(&Qs[(16 * b + r16) * LD + 16 * g + 4 * quad]);
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int b = 0; b < 4; ++b) o[b] = mfma_f32(q[b][e], t.s[g][e], o[b]);
      }
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) o[b][e] *= expf(static_cast<float>(As[16 * b + 4 * quad + e]));
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      f32x4 p[4];
#pragma unroll
      for (int b = k; b < 4; ++b) p[b] = *reinterpret_cast<const f32x4*>(&Ps[(16 * b + r16) * kMatLd + 16 * k + 4 * quad]);
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int b = k; b < 4; ++b) o[b] = mfma_f32(p[b][e], t.u[k][e], o[b]);
    }
    if (c < vdim) {
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int i = 16 * b + 4 * quad + e;
          if (i < n) {
            float v = o[b][e];
            if (!DELTA && skip != nullptr) v = fmaf(d_skip, t.u[b][e], v);
            out[(static_cast<int64_t>(t0 + i) * heads + h) * vdim + c] = v;
          }
        }
    }
  };
  for (int strip = w; strip < vpad / 16; strip += 4) {
    Strip t;
    fetch(t, strip);
    compute(t, strip);
  }
}

// ---- gate, then norm in equal parts of a row -----------------------------------------------------------------
// out[t, i] = y silu(z) / sqrt(mean over the element's part of (y silu(z))^2 + eps) * weight[i], z = p[t, gate_column + i].
// One workgroup per (token, part).
template <typename T>
__global__ __launch_bounds__(256) void gate_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ p,
                                                              int width, int gate_column, T* __restrict__ out, int inner,
                                                              int part, float eps, const void* __restrict__ weight,
                                                              int weight_is_f32) {
  __shared__ float scratch[16];
  const int64_t t = blockIdx.x;
  const int at = blockIdx.y * part;
  const float* yr = y + t * inner + at;
  const float* zr = p + t * width + gate_column + at;
  constexpr int kKeep = 8;  // products a thread keeps between the statistics and the result
  float kept[kKeep];
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < kKeep; ++u) {
    const int i = threadIdx.x + u * 256;
    kept[u] = i < part ? yr[i] * silu_f32(zr[i]) : 0.f;
    ss = fmaf(kept[u], kept[u], ss);
  }
  for (int i = threadIdx.x + kKeep * 256; i < part; i += 256) {
    const float v = yr[i] * silu_f32(zr[i]);
    ss = fmaf(v, v, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(part) + eps);
  T* dst = out + t * inner + at;
#pragma unroll
  for (int u = 0; u < kKeep; ++u) {
    const int i = threadIdx.x + u * 256;
    if (i < part) dst[i] = from_f32<T>(kept[u] * inv * load_as_f32(weight, at + i, weight_is_f32));
  }
  for (int i = threadIdx.x + kKeep * 256; i < part; i += 256)
    dst[i] = from_f32<T>(yr[i] * silu_f32(zr[i]) * inv * load_as_f32(weight, at + i, weight_is_f32));
}

}  // namespace
}  // namespace mlr

using namespace mlr;

extern "C" {

int mlr_conv_gates(const float* projected, int width, int column, const float* taps, const float* bias, float* state,
                   int state_rows, const int* read_rows, const int* write_rows, const int* token_entry, const int* cu_q,
                   const int* q_starts, float* out, float* gates, int channels, int n_taps, int unit_heads, int unit_dim,
                   int scaled_heads, float unit_scale, const float* rate, const float* dt_bias, int heads,
                   int step_column, int write_column, int tokens, hipStream_t stream) {
  MLR_REQUIRE(projected && taps && token_entry && cu_q && q_starts && out && gates && rate && dt_bias, "null pointer");
  MLR_REQUIRE(tokens > 0 && channels > 0 && n_taps > 0 && heads > 0, "sizes must be > 0");
  MLR_REQUIRE(n_taps == 1 || (state && read_rows && write_rows && state_rows > 0), "several taps carry inputs");
  MLR_REQUIRE(unit_heads >= 0 && (unit_heads == 0 || (unit_dim > 0 && unit_dim <= 256)), "unit heads of 1 to 256 channels");
  MLR_REQUIRE(static_cast<int64_t>(unit_heads) * unit_dim <= channels && scaled_heads <= unit_heads, "unit heads lie within the channels");
  MLR_REQUIRE(column >= 0 && column + channels <= width && step_column >= 0 && step_column + heads <= width &&
                  (write_column < 0 || write_column + heads <= width),
              "the projected rows do not hold what the columns name");
  const int plain_jobs = (channels - unit_heads * unit_dim + kPlainChannels - 1) / kPlainChannels;
  const int jobs = unit_heads + plain_jobs + 1;
  MLR_REQUIRE((jobs + 3) / 4 < 65536, "too many channels for one launch");
  const dim3 grid(tokens, (jobs + 3) / 4);
#define MLR_CONV(TAPS)                                                                                             \
  conv_gates_kernel<TAPS><<<grid, 256, 0, stream>>>(projected, width, column, taps, bias, state, read_rows, write_rows, \
                                                    token_entry, cu_q, q_starts, out, gates, channels, n_taps,      \
                                                    unit_heads, unit_dim, scaled_heads, unit_scale, rate, dt_bias,  \
                                                    heads, step_column, write_column, plain_jobs)
  if (n_taps == 2)
    MLR_CONV(2);
  else if (n_taps == 3)
    MLR_CONV(3);
  else if (n_taps == 4)
    MLR_CONV(4);
  else
    MLR_CONV(0);
#undef MLR_CONV
  MLR_LAUNCH_CHECK();
  return 0;
}

static int padded_rows(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : 128; }

// Floats of scratch memory that mlr_decay_scan needs to go by chunks (0: it will not go that way).
int64_t mlr_decay_scan_scratch(int tokens, int entries, int heads, int key_heads, int dim, int vdim, int delta) {
  if (tokens <= 0 || entries <= 0 || heads <= 0 || key_heads <= 0 || dim <= 0 || vdim <= 0 || dim > 128) return 0;
  const int64_t cells = (static_cast<int64_t>(tokens) / kChunk + entries) * heads;
  return cells * scratch_floats_per_chunk(padded_rows(dim), (vdim + 15) / 16 * 16, delta);
}

int mlr_decay_scan(const float* x, int channels, int q_off, int k_off, int v_off, const float* gates, float* state,
                   int state_rows, const int* read_rows, const int* write_rows, const int* cu_q, const int* q_starts,
                   const float* skip, float* out, int entries, int heads, int key_heads, int dim, int vdim, int tokens,
                   int delta, float* scratch, int64_t scratch_floats, hipStream_t stream) {
  MLR_REQUIRE(x && gates && state && read_rows && write_rows && cu_q && q_starts && out, "null pointer");
  MLR_REQUIRE(entries > 0 && heads > 0 && heads < 65536 && key_heads > 0 && heads % key_heads == 0 && vdim > 0 &&
                  state_rows > 0 && tokens > 0,
              "bad sizes");
  MLR_REQUIRE(dim > 0 && dim <= 256, "states of up to 256 rows");
  MLR_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + key_heads * dim <= channels &&
                  k_off + key_heads * dim <= channels && v_off + heads * vdim <= channels,
              "the rows do not hold what the offsets name");
  MLR_REQUIRE(skip == nullptr || !delta, "the delta rule's scan adds no skip");
  const int64_t needed = mlr_decay_scan_scratch(tokens, entries, heads, key_heads, dim, vdim, delta);
  if (scratch != nullptr && needed > 0) {
    MLR_REQUIRE(scratch_floats >= needed, "the scratch memory is too small");
    MLR_REQUIRE(entries < 65536, "too many entries for one launch");
    const int chunks = tokens / kChunk + entries;
    const int dp = padded_rows(dim), vpad = (vdim + 15) / 16 * 16;
    const ChunkScratch s = chunk_scratch(scratch, static_cast<int64_t>(chunks) * heads, dp, vpad, delta);
#define MLR_CHUNKS(DP, DELTA)                                                                                          \
  do {                                                                                                               \
    constexpr int kLds = 2 * kChunk * (DP + 8) * 4;                                                                  \
    constexpr int kApplyLds = kLds > (kChunk * (DP + 8) + kChunk * kMatLd) * 4 ? kLds : (kChunk * (DP + 8) + kChunk * kMatLd) * 4; \
    static bool configured = false;                                                                                  \
    if (!configured) {                                                                                               \
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(decay_apply_kernel<DP, DELTA>),          \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, kApplyLds);               \
      if (e != hipSuccess) {                                                                                         \
        set_error(std::string("mlr_decay_scan: cannot raise the LDS limit: ") + hipGetErrorString(e));               \
        return -1;                                                                                                   \
      }                                                                                                              \
      configured = true;                                                                                             \
    }                                                                                                                \
    decay_local_kernel<DP, DELTA><<<dim3(chunks, heads), 256, 0, stream>>>(x, channels, k_off, v_off, gates, cu_q,    \
                                                                           entries, heads, key_heads, dim, vdim, s); \
    MLR_LAUNCH_CHECK();                                                                                              \
    if constexpr (DELTA)                                                                                             \
      delta_carry_kernel<DP><<<static_cast<unsigned>((entries * heads + kDies - 1) / kDies * kDies * (vpad / 16)), 256, 0, \
                               stream>>>(state, read_rows, write_rows, cu_q, q_starts, entries, heads, dim, vdim, s); \
    else                                                                                                             \
      plain_carry_kernel<<<dim3(entries, heads, (dp * vpad + 255) / 256), 256, 0, stream>>>(                         \
          state, read_rows, write_rows, cu_q, q_starts, heads, dim, vdim, s);                                        \
    MLR_LAUNCH_CHECK();                                                                                              \
    decay_apply_kernel<DP, DELTA><<<dim3(chunks, heads), 256, kApplyLds, stream>>>(                                   \
        x, channels, q_off, k_off, v_off, gates, cu_q, q_starts, skip, out, entries, heads, key_heads, dim, vdim, s); \
    MLR_LAUNCH_CHECK();                                                                                              \
  } while (0)
#define MLR_CHUNKS_SIZED(DELTA) \
  do {                          \
    if (dp == 32)               \
      MLR_CHUNKS(32, DELTA);    \
    else if (dp == 64)          \
      MLR_CHUNKS(64, DELTA);    \
    else                        \
      MLR_CHUNKS(128, DELTA);   \
  } while (0)
    if (delta)
      MLR_CHUNKS_SIZED(true);
    else
      MLR_CHUNKS_SIZED(false);
#undef MLR_CHUNKS_SIZED
#undef MLR_CHUNKS
    return 0;
  }
#define MLR_WALK(R, DELTA)                                                                                        \
  decay_walk_kernel<R, DELTA><<<dim3(entries, heads, (vdim + 63) / 64), 256, 0, stream>>>(                         \
      x, channels, q_off, k_off, v_off, gates, state, read_rows, write_rows, cu_q, q_starts, skip, out, heads,    \
      key_heads, dim, vdim)
#define MLR_WALK_SIZED(DELTA) \
  do {                        \
    if (dim <= 64)            \
      MLR_WALK(16, DELTA);    \
    else if (dim <= 128)      \
      MLR_WALK(32, DELTA);    \
    else                      \
      MLR_WALK(64, DELTA);    \
  } while (0)
  if (delta)
    MLR_WALK_SIZED(true);
  else
    MLR_WALK_SIZED(false);
#undef MLR_WALK_SIZED
#undef MLR_WALK
  MLR_LAUNCH_CHECK();
  return 0;
}

// Convolution, gates and scan of a step of single tokens (entry e is token e) in one kernel: mlr_conv_gates followed by
// mlr_decay_scan, for up to 4 taps.  With `delta` q and k are unit heads (q times unit_scale), without it there are none.
int mlr_decay_step(const float* projected, int width, int column, const float* taps, const float* bias, float* carried,
                   int carried_rows, const int* carried_read, const int* carried_write, int channels, int n_taps,
                   float unit_scale, const float* rate, const float* dt_bias, int step_column, int write_column, int q_off,
                   int k_off, int v_off, float* state, int state_rows, const int* read_rows, const int* write_rows,
                   const int* q_starts, const float* skip, float* out, int entries, int heads, int key_heads, int dim,
                   int vdim, int delta, hipStream_t stream) {
  MLR_REQUIRE(projected && taps && rate && dt_bias && state && read_rows && write_rows && q_starts && out, "null pointer");
  MLR_REQUIRE(n_taps > 0 && n_taps <= kStepTaps, "up to 4 taps");
  MLR_REQUIRE(n_taps == 1 || (carried && carried_read && carried_write && carried_rows > 0), "several taps carry inputs");
  MLR_REQUIRE(entries > 0 && heads > 0 && heads < 65536 && key_heads > 0 && heads % key_heads == 0 && vdim > 0 && state_rows > 0,
              "bad sizes");
  MLR_REQUIRE(dim > 0 && dim <= 256, "states of up to 256 rows");
  MLR_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + key_heads * dim <= channels &&
                  k_off + key_heads * dim <= channels && v_off + heads * vdim <= channels &&
                  channels == 2 * key_heads * dim + heads * vdim,
              "the channels are those of q, k and v");
  MLR_REQUIRE(column >= 0 && column + channels <= width && step_column >= 0 && step_column + heads <= width &&
                  (write_column < 0 || write_column + heads <= width),
              "the projected rows do not hold what the columns name");
  const StepConv in{projected, width, column, n_taps, taps, bias, carried, carried_read, carried_write, rate, dt_bias,
                    step_column, write_column, unit_scale};
#define MLR_STEP(R, DELTA)                                                                                          \
  decay_step_kernel<R, DELTA><<<dim3(entries, heads, (vdim + 63) / 64), 256, 0, stream>>>(                          \
      in, channels, q_off, k_off, v_off, state, read_rows, write_rows, q_starts, skip, out, heads, key_heads, dim, vdim)
#define MLR_STEP_SIZED(DELTA) \
  do {                        \
    if (dim <= 64)            \
      MLR_STEP(16, DELTA);    \
    else if (dim <= 128)      \
      MLR_STEP(32, DELTA);    \
    else                      \
      MLR_STEP(64, DELTA);    \
  } while (0)
  if (delta)
    MLR_STEP_SIZED(true);
  else
    MLR_STEP_SIZED(false);
#undef MLR_STEP_SIZED
#undef MLR_STEP
  MLR_LAUNCH_CHECK();
  return 0;
}

int mlr_gate_group_norm(const float* y, const float* projected, int width, int gate_column, void* out, int dtype,
                        int tokens, int inner, int groups, float eps, const void* weight, int weight_is_f32,
                        hipStream_t stream) {
  MLR_REQUIRE(y && projected && out && weight, "null pointer");
  MLR_REQUIRE(tokens > 0 && inner > 0 && groups > 0 && inner % groups == 0 && groups < 65536, "parts of a row must be equal");
  MLR_REQUIRE(gate_column >= 0 && gate_column + inner <= width, "the projected rows do not hold the gate");
  MLR_REQUIRE(dtype == kF32 || dtype == kBF16, "dtype must be 0 (float32) or 1 (bfloat16)");
  const dim3 grid(tokens, groups);
  if (dtype == kF32)
    gate_group_norm_kernel<float><<<grid, 256, 0, stream>>>(y, projected, width, gate_column, static_cast<float*>(out),
                                                            inner, inner / groups, eps, weight, weight_is_f32);
  else
    gate_group_norm_kernel<bf16><<<grid, 256, 0, stream>>>(y, projected, width, gate_column, static_cast<bf16*>(out), inner,
                                                           inner / groups, eps, weight, weight_is_f32);
  MLR_LAUNCH_CHECK();
  return 0;
}

}  // extern "C"
