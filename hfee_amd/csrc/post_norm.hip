// Row-wise steps of blocks that norm the sum of the stream and a sub-layer's result (the norm stands behind the
// addition), and of a mixer's input that is mixed with the token before it:
//
//   post_norm:     v = alpha x[r] + a y[r] + b y2[r] (y2 optional);  x[r] = v / sqrt(mean(v^2) + eps) * w, and, if
//                  asked, in the same launch the next sub-layer's input: x[r] in the engine's dtype, or, where every
//                  row is a sequence's only token of the step, the shifted input as below with the slot's row
//   token_shift:   next[t] = x[t] + (x[t - 1] - x[t]) * mu, element by element, with x[t - 1] the row before in the same
//                  sequence; before a portion's first row stands the row that the step before left in the
//                  request's slot (zeros at a sequence's start), and the portion's last row is left there
//   softcap:       x = cap * tanh(x / cap), in place (logits)
//
// All sums in float32, one workgroup a row, a fixed order of additions (which depends on the row's width and
// alignment only, never on the other rows of the step).
#include "common.h"

using namespace hfee;

namespace {

// What a row becomes for the sub-layer that reads it next.
struct NextInput {
  const float* shift;        // mu [d], or null: the row as it is
  float* state;              // [slots][d] float32, with shift
  const int* segment_slots;  // row r is the only token of segment r
};

__device__ __forceinline__ float joined(const float* x, const float* y, const float* y2, float alpha, float a, float b, int64_t j) {
  const float v = fmaf(alpha, x[j], a * y[j]);
  return y2 != nullptr ? fmaf(b, y2[j], v) : v;
}

template <typename TN>
__global__ __launch_bounds__(256) void post_norm_kernel(float* __restrict__ x, const float* __restrict__ y,
                                                        const float* __restrict__ y2, float alpha, float a, float b,
                                                        const float* __restrict__ w, float eps, TN* __restrict__ next,
                                                        NextInput in, int d) {
  __shared__ float scratch[16];
  const int64_t r = blockIdx.x, at = r * d;
  float ss = 0.f;
  for (int j = threadIdx.x; j < d; j += blockDim.x) {
    const float v = joined(x, y, y2, alpha, a, b, at + j);
    ss = fmaf(v, v, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)d + eps);
  float* state = in.shift != nullptr ? in.state + (int64_t)in.segment_slots[r] * d : nullptr;
  for (int j = threadIdx.x; j < d; j += blockDim.x) {
    const float v = joined(x, y, y2, alpha, a, b, at + j) * inv * w[j];
    x[at + j] = v;
    if (next == nullptr) continue;
    if (in.shift != nullptr) {
      next[at + j] = from_float<TN>(fmaf(state[j] - v, in.shift[j], v));
      state[j] = v;
    } else {
      next[at + j] = from_float<TN>(v);
    }
  }
}

// The same for rows of up to 4 * K * blockDim values that are whole groups of four: a thread asks for all it needs
// of the row at once and keeps the sum's row in registers between the two passes.
template <typename TN, int K>
__global__ __launch_bounds__(1024) void post_norm_held_kernel(float* __restrict__ x, const float* __restrict__ y,
                                                              const float* __restrict__ y2, float alpha, float a, float b,
                                                              const float* __restrict__ w, float eps, TN* __restrict__ next,
                                                              NextInput in, int d) {
  __shared__ float scratch[16];
  const int64_t r = blockIdx.x, at = r * d;
  float* state = in.shift != nullptr ? in.state + (int64_t)in.segment_slots[r] * d : nullptr;
  float v[K][4], ws[K][4], before[K][4], mu[K][4];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int j = (k * blockDim.x + threadIdx.x) * 4;
    const bool mine = j < d;
    const int jj = mine ? j : 0;
    float first[4], second[4];
    load4<float>(v[k], x + at + jj);
    load4<float>(first, y + at + jj);
    load4<float>(ws[k], w + jj);
    if (y2 != nullptr) load4<float>(second, y2 + at + jj);
    if (in.shift != nullptr) {
      load4<float>(before[k], state + jj);
      load4<float>(mu[k], in.shift + jj);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float t = fmaf(alpha, v[k][i], a * first[i]);
      if (y2 != nullptr) t = fmaf(b, second[i], t);
      v[k][i] = mine ? t : 0.f;
      ss = fmaf(v[k][i], v[k][i], ss);
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)d + eps);
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int j = (k * blockDim.x + threadIdx.x) * 4;
    if (j >= d) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[k][i] = v[k][i] * inv * ws[k][i];
    store4<float>(x + at + j, v[k]);
    if (next == nullptr) continue;
    if (in.shift != nullptr) {
      store4<float>(state + j, v[k]);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[k][i] = fmaf(before[k][i] - v[k][i], mu[k][i], v[k][i]);
    }
    store4<TN>(next + at + j, v[k]);
  }
}

// grid (rows, parts of the columns).  The thread that makes column c of a portion's first row is the only one that
// touches column c of the slot's row: it reads what the step before left there, then leaves the portion's last row.
template <typename TN, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(TN* __restrict__ next, const float* __restrict__ x, int d,
                                                          float* __restrict__ state, const float* __restrict__ mu,
                                                          const int* __restrict__ token_segment,
                                                          const int* __restrict__ segment_rows,
                                                          const int* __restrict__ segment_lengths,
                                                          const int* __restrict__ segment_slots) {
  const int t = blockIdx.x, seg = token_segment[t], row0 = segment_rows[seg];
  float* st = state + (int64_t)segment_slots[seg] * d;
  const float* xr = x + (int64_t)t * d;
  const float* last = x + (int64_t)(row0 + segment_lengths[seg] - 1) * d;
  for (int c = (blockIdx.y * blockDim.x + threadIdx.x) * V; c < d; c += gridDim.y * blockDim.x * V) {
    const float* from = t == row0 ? st + c : xr - d + c;
    if constexpr (V == 4) {
      float now[4], before[4], m[4], keep[4];
      load4<float>(now, xr + c);
      load4<float>(before, from);
      load4<float>(m, mu + c);
      if (t == row0) {
        load4<float>(keep, last + c);
        store4<float>(st + c, keep);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) now[i] = fmaf(before[i] - now[i], m[i], now[i]);
      store4<TN>(next + (int64_t)t * d + c, now);
    } else {
      const float now = xr[c], before = *from;
      if (t == row0) st[c] = last[c];
      next[(int64_t)t * d + c] = from_float<TN>(fmaf(before - now, mu[c], now));
    }
  }
}

__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ x, float cap, int64_t count) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < count) x[i] = cap * tanhf(x[i] / cap);
}

bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

}  // namespace

// x, y, y2: float32 [n, d] contiguous; w, shift: float32 [d]; next (or null): [n, d] in next_dtype (0 float32, 1
// bfloat16).  With shift, row r of the step is the only token of segment r.
HFEE_API int hfee_post_norm(float* x, const float* y, float a, const float* y2, float b, float alpha, const float* w, float eps,
                            void* next, int next_dtype, const float* shift, float* state, const int* segment_slots, int n,
                            int d, hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && d > 0 && x != nullptr && y != nullptr && w != nullptr && eps >= 0.f, "post_norm: bad arguments");
  HFEE_REQUIRE(next_dtype == 0 || next_dtype == 1, "post_norm: unknown dtype %d", next_dtype);
  HFEE_REQUIRE(shift == nullptr || (next != nullptr && state != nullptr && segment_slots != nullptr),
               "post_norm: a shifted input comes with its rows, the states and the slots");
  if (n == 0) return 0;
  const NextInput in{shift, state, segment_slots};
  const bool held = d % 4 == 0 && d <= 16384 && aligned16(x) && aligned16(y) && aligned16(y2) && aligned16(w) && aligned16(next) &&
                    aligned16(shift) && aligned16(state);
  if (!held) {
    if (next_dtype == 0) post_norm_kernel<float><<<n, 256, 0, stream>>>(x, y, y2, alpha, a, b, w, eps, (float*)next, in, d);
    else post_norm_kernel<bf16_t><<<n, 256, 0, stream>>>(x, y, y2, alpha, a, b, w, eps, (bf16_t*)next, in, d);
    HFEE_CHECK_LAUNCH("post_norm");
    return 0;
  }
  const int quads = d / 4, nv = quads <= 1024 ? 1 : quads <= 2048 ? 2 : 4;
  int threads = ((quads + nv - 1) / nv + 63) / 64 * 64;
  if (threads > 1024) threads = 1024;
#define LAUNCH(TN, K)                                                                                                \
  post_norm_held_kernel<TN, K><<<n, threads, 0, stream>>>(x, y, y2, alpha, a, b, w, eps, (TN*)next, in, d)
#define PICK(TN)                                                                                                     \
  if (nv == 1) LAUNCH(TN, 1); else if (nv == 2) LAUNCH(TN, 2); else LAUNCH(TN, 4)
  if (next_dtype == 0) { PICK(float); } else { PICK(bf16_t); }
#undef PICK
#undef LAUNCH
  HFEE_CHECK_LAUNCH("post_norm");
  return 0;
}

HFEE_API int hfee_token_shift(void* next, int next_dtype, const float* x, float* state, const float* mu,
                              const int* token_segment, const int* segment_rows, const int* segment_lengths,
                              const int* segment_slots, int n, int d, hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && d > 0 && next != nullptr && x != nullptr && state != nullptr && mu != nullptr, "token_shift: bad arguments");
  HFEE_REQUIRE(token_segment != nullptr && segment_rows != nullptr && segment_lengths != nullptr && segment_slots != nullptr,
               "token_shift: the step's segments are missing");
  HFEE_REQUIRE(next_dtype == 0 || next_dtype == 1, "token_shift: unknown dtype %d", next_dtype);
  HFEE_REQUIRE(next != (const void*)x, "token_shift: the shifted rows cannot lie where the rows are");
  if (n == 0) return 0;
  const bool wide = d % 4 == 0 && aligned16(next) && aligned16(x) && aligned16(state) && aligned16(mu);
  int parts = (d + 256 * (wide ? 4 : 1) - 1) / (256 * (wide ? 4 : 1));
  if (parts > 64) parts = 64;
  const dim3 grid(n, parts);
#define LAUNCH(TN, V)                                                                                                \
  token_shift_kernel<TN, V><<<grid, 256, 0, stream>>>((TN*)next, x, d, state, mu, token_segment, segment_rows,       \
                                                      segment_lengths, segment_slots)
  if (next_dtype == 0) { if (wide) LAUNCH(float, 4); else LAUNCH(float, 1); }
  else { if (wide) LAUNCH(bf16_t, 4); else LAUNCH(bf16_t, 1); }
#undef LAUNCH
  HFEE_CHECK_LAUNCH("token_shift");
  return 0;
}

// x (float32, contiguous) = cap * tanh(x / cap).
HFEE_API int hfee_softcap(float* x, float cap, int64_t count, hipStream_t stream) {
  HFEE_REQUIRE(count >= 0 && (count + 255) / 256 <= 0x7fffffff && x != nullptr && cap > 0.f, "softcap: bad arguments");
  if (count == 0) return 0;
  softcap_kernel<<<(unsigned)((count + 255) / 256), 256, 0, stream>>>(x, cap, count);
  HFEE_CHECK_LAUNCH("softcap");
  return 0;
}
