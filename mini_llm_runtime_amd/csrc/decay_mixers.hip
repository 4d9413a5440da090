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

int64_t mlr_decay_scan_scratch(int tokens, int entries, int heads, int key_heads, int dim, int vdim, int delta) { return 0; }

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
