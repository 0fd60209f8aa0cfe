// Row-wise steps around norms that cut a row into groups, and what joins the residual stream in the launch that norms
// it next:
//
//   group_norm:     out[r] = x[rows[r] or r], cut into `groups` equal parts, each divided by its own
//                   sqrt(mean(part^2) + eps), the whole times w
//   pair_norm_add:  x[r] += a y[r] / sqrt(mean(y[r]^2) + e) wy + b y2[r] / sqrt(mean(y2[r]^2) + e) wy2    (two mixers side
//                   by side, each result normed over the row with a weight of its own)
//   experts_join:   x[r] += sigmoid(gate[r]) s[r] + sum_j w[r][j] (expert j of the row is a real one ? its output : h[r]):
//                   the routed experts' outputs (a row a pair, or already summed), the experts that hand on their
//                   input, and an expert that every token uses behind a gate of one number a token
//   poly_norm:      out = a N(z) + b N(z^2) + c N(z^3) + e, powers element by element, N(v) = v / sqrt(mean(v^2) + eps) over the row
//
// pair_norm_add and experts_join go on, if asked, with the group norm of the new row for what follows.  One workgroup a
// row, all sums in float32, a fixed order of additions (which depends on the row's width, the groups and the alignment
// only, never on the other rows of the step).  Rows of whole groups of four that fit a workgroup's registers are read
// once, sixteen bytes a load; other rows go through loops.
#include "common.h"

using namespace hfee;

namespace {

struct NextNorm {
  void* out;             // [n, d] in the engine's dtype, contiguous, or null
  const float* w;        // [d]
  float eps;
  int groups;
};

constexpr int kSums = 16;      // waves of a workgroup at most

// Sums of N numbers a thread over the workgroup; scratch: N * kSums floats.
template <int N>
__device__ __forceinline__ void block_sums(float (&v)[N], float* scratch) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = (blockDim.x + 63) >> 6;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = wave_sum(v[i]);
  __syncthreads();
  if (lane == 0) {
#pragma unroll
    for (int i = 0; i < N; ++i) scratch[i * kSums + wave] = v[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < N; ++i) {
    float total = 0.f;
    for (int w = 0; w < waves; ++w) total += scratch[i * kSums + w];
    v[i] = total;
  }
}

// The group norm of a row that the workgroup holds in registers: thread t has the fours k * blockDim.x + t (zeros
// behind the row's end).  lds: d / 4 + groups floats, not read by anyone when this is called.
template <typename T, int K>
__device__ __forceinline__ void norm_held_row(const float (&x)[K][4], T* out, const float* w, float eps, int groups, int d, float* lds) {
  const int fours = d >> 2, each = fours / groups, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int waves = blockDim.x >> 6;
  float ss[K], ws[K][4];
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int q = k * blockDim.x + threadIdx.x;
    load4<float>(ws[k], w + (q < fours ? q : 0) * 4);
    ss[k] = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) ss[k] = fmaf(x[k][i], x[k][i], ss[k]);
  }
  const float width = (float)(each * 4);
  if (each % 64 == 0) {      // (the 64 fours of a wave belong to one group)
#pragma unroll
    for (int k = 0; k < K; ++k) {
      ss[k] = wave_sum(ss[k]);
      if (lane == 0) lds[k * waves + wave] = ss[k];
    }
    __syncthreads();
    const int parts = each / 64;
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int q = k * blockDim.x + threadIdx.x;
      if (q >= fours) continue;
      const float* from = lds + q / each * parts;
      float total = 0.f;
      for (int i = 0; i < parts; ++i) total += from[i];
      ss[k] = 1.0f / sqrtf(total / width + eps);
    }
  } else {
    float* inv = lds + fours;
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int q = k * blockDim.x + threadIdx.x;
      if (q < fours) lds[q] = ss[k];
    }
    __syncthreads();
    for (int g = wave; g < groups; g += waves) {
      float total = 0.f;
      for (int q = lane; q < each; q += 64) total += lds[g * each + q];
      total = wave_sum(total);
      if (lane == 0) inv[g] = 1.0f / sqrtf(total / width + eps);
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int q = k * blockDim.x + threadIdx.x;
      if (q < fours) ss[k] = inv[q / each];
    }
  }
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int q = k * blockDim.x + threadIdx.x;
    if (q >= fours) continue;
    float y[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] = x[k][i] * ss[k] * ws[k][i];
    store4<T>(out + q * 4, y);
  }
}

// The same from memory (x may have been written by the workgroup's other threads).  scratch: 16 floats.
template <typename T>
__device__ __forceinline__ void norm_stored_row(const float* x, T* out, const float* w, float eps, int groups, int d, float* scratch) {
  const int each = d / groups;
  __syncthreads();
  for (int j0 = 0; j0 < d; j0 += each) {
    float ss = 0.f;
    for (int j = j0 + threadIdx.x; j < j0 + each; j += blockDim.x) ss = fmaf(x[j], x[j], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)each + eps);
    for (int j = j0 + threadIdx.x; j < j0 + each; j += blockDim.x) out[j] = from_float<T>(x[j] * inv * w[j]);
  }
}

template <int K>
__device__ __forceinline__ void load_row(float (&v)[K][4], const float* p, int fours) {
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int q = k * blockDim.x + threadIdx.x;
    load4<float>(v[k], p + (q < fours ? q : 0) * 4);
    if (q >= fours) v[k][0] = v[k][1] = v[k][2] = v[k][3] = 0.f;
  }
}

template <int K>
__device__ __forceinline__ void store_row(float* p, const float (&v)[K][4], int fours) {
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int q = k * blockDim.x + threadIdx.x;
    if (q < fours) store4<float>(p + q * 4, v[k]);
  }
}

extern __shared__ __attribute__((aligned(16))) float row_lds[];

template <typename T, int K>      // K 0: loops
__global__ __launch_bounds__(1024) void group_norm_kernel(const float* __restrict__ x, const int* __restrict__ rows, NextNorm to, int d) {
  __shared__ float scratch[kSums];
  const int64_t r = blockIdx.x;
  const float* xr = x + (int64_t)(rows != nullptr ? rows[r] : r) * d;
  T* out = (T*)to.out + r * d;
  if constexpr (K == 0) {
    norm_stored_row<T>(xr, out, to.w, to.eps, to.groups, d, scratch);
  } else {
    float v[K][4];
    load_row<K>(v, xr, d >> 2);
    norm_held_row<T, K>(v, out, to.w, to.eps, to.groups, d, row_lds);
  }
}

template <typename T, int K>
__global__ __launch_bounds__(1024) void pair_norm_add_kernel(float* x, const float* __restrict__ y, const float* __restrict__ y2,
                                                             const float* __restrict__ wy, const float* __restrict__ wy2, float a,
                                                             float b, float eps, NextNorm to, int d) {
  __shared__ float scratch[2 * kSums];
  const int64_t r = blockIdx.x;
  float* xr = x + r * d;
  float ss[2] = {0.f, 0.f};
  if constexpr (K == 0) {
    for (int j = threadIdx.x; j < d; j += blockDim.x) {
      ss[0] = fmaf(y[r * d + j], y[r * d + j], ss[0]);
      ss[1] = fmaf(y2[r * d + j], y2[r * d + j], ss[1]);
    }
    block_sums<2>(ss, scratch);
    const float ia = a / sqrtf(ss[0] / (float)d + eps), ib = b / sqrtf(ss[1] / (float)d + eps);
    for (int j = threadIdx.x; j < d; j += blockDim.x) xr[j] += fmaf(y[r * d + j] * ia, wy[j], y2[r * d + j] * ib * wy2[j]);
    if (to.out != nullptr) norm_stored_row<T>(xr, (T*)to.out + r * d, to.w, to.eps, to.groups, d, scratch);
  } else {
    const int fours = d >> 2;
    float v[K][4], first[K][4], second[K][4], w1[K][4], w2[K][4];
    load_row<K>(first, y + r * d, fours);
    load_row<K>(second, y2 + r * d, fours);
    load_row<K>(v, xr, fours);
    load_row<K>(w1, wy, fours);
    load_row<K>(w2, wy2, fours);
#pragma unroll
    for (int k = 0; k < K; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ss[0] = fmaf(first[k][i], first[k][i], ss[0]);
        ss[1] = fmaf(second[k][i], second[k][i], ss[1]);
      }
    block_sums<2>(ss, scratch);
    const float ia = a / sqrtf(ss[0] / (float)d + eps), ib = b / sqrtf(ss[1] / (float)d + eps);
#pragma unroll
    for (int k = 0; k < K; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) v[k][i] += fmaf(first[k][i] * ia, w1[k][i], second[k][i] * ib * w2[k][i]);
    store_row<K>(xr, v, fours);
    if (to.out != nullptr) norm_held_row<T, K>(v, (T*)to.out + r * d, to.w, to.eps, to.groups, d, row_lds);
  }
}

struct JoinArgs {
  float* x;
  const float* y;              // [n * top, d], a row a (token, expert) pair (rows of other than real experts are not
                               // looked at), or [n, d] with `summed`
  int summed;
  const int* chosen;           // [n, top]
  const float* weights;        // [n, top]
  int top, experts;            // experts at and beyond `experts` hand on their input
  const void* h;               // [n, d] in the engine's dtype, rows ldh apart
  int64_t ldh;
  const float* shared;         // [n, d] or null
  const float* gate;           // one number a row (before the sigmoid), ldg apart, or null (then shared counts as it is)
  int64_t ldg;
};

template <typename T, int K>
__global__ __launch_bounds__(1024) void experts_join_kernel(JoinArgs p, NextNorm to, int d) {
  __shared__ float scratch[kSums];
  const int64_t r = blockIdx.x;
  float* xr = p.x + r * d;
  const int* chosen = p.chosen + r * p.top;
  const float* weights = p.weights + r * p.top;
  float handed_on = 0.f;
  for (int j = 0; j < p.top; ++j)
    if (chosen[j] >= p.experts) handed_on += weights[j];
  const float g = p.gate != nullptr ? 1.0f / (1.0f + expf(-p.gate[r * p.ldg])) : 1.0f;
  const T* h = (const T*)p.h + r * p.ldh;
  if constexpr (K == 0) {
    for (int c = threadIdx.x; c < d; c += blockDim.x) {
      float v = 0.f;
      if (p.summed) v = p.y[r * d + c];
      else
        for (int j = 0; j < p.top; ++j)
          if (chosen[j] < p.experts) v = fmaf(p.y[(r * p.top + j) * d + c], weights[j], v);
      if (handed_on != 0.f) v = fmaf(handed_on, to_float<T>(h[c]), v);
      if (p.shared != nullptr) v = fmaf(g, p.shared[r * d + c], v);
      xr[c] += v;
    }
    if (to.out != nullptr) norm_stored_row<T>(xr, (T*)to.out + r * d, to.w, to.eps, to.groups, d, scratch);
  } else {
    const int fours = d >> 2;
    float v[K][4], one[K][4], sum[K][4];
    load_row<K>(v, xr, fours);
    if (p.summed) {
      load_row<K>(sum, p.y + r * d, fours);
    } else {
#pragma unroll
      for (int k = 0; k < K; ++k) sum[k][0] = sum[k][1] = sum[k][2] = sum[k][3] = 0.f;
      for (int j = 0; j < p.top; ++j) {
        if (chosen[j] >= p.experts) continue;
        const float w = weights[j];
        load_row<K>(one, p.y + (r * p.top + j) * d, fours);
#pragma unroll
        for (int k = 0; k < K; ++k)
#pragma unroll
          for (int i = 0; i < 4; ++i) sum[k][i] = fmaf(one[k][i], w, sum[k][i]);
      }
    }
    if (handed_on != 0.f) {
#pragma unroll
      for (int k = 0; k < K; ++k) {
        const int q = k * blockDim.x + threadIdx.x;
        float hv[4];
        load4<T>(hv, h + (q < fours ? q : 0) * 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) sum[k][i] = fmaf(handed_on, hv[i], sum[k][i]);
      }
    }
    if (p.shared != nullptr) {
      load_row<K>(one, p.shared + r * d, fours);
#pragma unroll
      for (int k = 0; k < K; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) sum[k][i] = fmaf(g, one[k][i], sum[k][i]);
    }
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const bool mine = k * blockDim.x + threadIdx.x < fours;
#pragma unroll
      for (int i = 0; i < 4; ++i) v[k][i] = mine ? v[k][i] + sum[k][i] : 0.f;
    }
    store_row<K>(xr, v, fours);
    if (to.out != nullptr) norm_held_row<T, K>(v, (T*)to.out + r * d, to.w, to.eps, to.groups, d, row_lds);
  }
}

// numbers: float32 [4] (a, b, c, e).  out may be z.
template <typename T, int K>
__global__ __launch_bounds__(1024) void poly_norm_kernel(T* out, int64_t ldo, const T* z, int64_t ldz, const float* __restrict__ numbers,
                                                         float eps, int d) {
  __shared__ float scratch[3 * kSums];
  const int64_t r = blockIdx.x;
  const T* zr = z + r * ldz;
  T* o = out + r * ldo;
  float ss[3] = {0.f, 0.f, 0.f};
  auto powers = [&](float v) {
    const float v2 = v * v, v3 = v2 * v;
    ss[0] += v2;
    ss[1] = fmaf(v2, v2, ss[1]);
    ss[2] = fmaf(v3, v3, ss[2]);
  };
  float held[K == 0 ? 1 : K][4];
  if constexpr (K == 0) {
    for (int j = threadIdx.x; j < d; j += blockDim.x) powers(to_float<T>(zr[j]));
  } else {
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int j = (k * blockDim.x + threadIdx.x) * 4;
      load4<T>(held[k], zr + (j < d ? j : 0));
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (j >= d) held[k][i] = 0.f;
        powers(held[k][i]);
      }
    }
  }
  block_sums<3>(ss, scratch);      // (its barriers stand between every read of the row and the writes: in place is fine)
  const float a = numbers[0] / sqrtf(ss[0] / (float)d + eps), b = numbers[1] / sqrtf(ss[1] / (float)d + eps),
              c = numbers[2] / sqrtf(ss[2] / (float)d + eps), e = numbers[3];
  auto value = [&](float v) { return fmaf(v, fmaf(v, fmaf(v, c, b), a), e); };
  if constexpr (K == 0) {
    for (int j = threadIdx.x; j < d; j += blockDim.x) o[j] = from_float<T>(value(to_float<T>(zr[j])));
  } else {
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int j = (k * blockDim.x + threadIdx.x) * 4;
      if (j >= d) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) held[k][i] = value(held[k][i]);
      store4<T>(o + j, held[k]);
    }
  }
}

bool aligned(const void* p, int to) { return (reinterpret_cast<uintptr_t>(p) & (uintptr_t)(to - 1)) == 0; }

// How a row of d values is held: fours a thread (0: not held), and the threads.
struct RowShape {
  int held, threads;
};
RowShape row_shape(bool fits, int d) {
  if (!fits || d % 4 != 0 || d > 32768) return {0, 256};
  const int fours = d / 4, held = fours <= 1024 ? 1 : fours <= 2048 ? 2 : fours <= 4096 ? 4 : 8;
  int threads = ((fours + held - 1) / held + 63) / 64 * 64;
  return {held, threads > 1024 ? 1024 : threads};
}
size_t norm_lds(const RowShape& s, const NextNorm& to, int d) {
  return s.held != 0 && to.out != nullptr ? (size_t)(d / 4 + to.groups) * sizeof(float) : 0;
}
bool next_fits(const NextNorm& to, int d) {
  return to.out == nullptr || (aligned(to.out, 16) && aligned(to.w, 16) && d / to.groups % 4 == 0);
}
int check_next(const NextNorm& to, int dtype, int d, const char* what) {
  if (dtype != 0 && dtype != 1) return fail("%s: unknown dtype %d", what, dtype);
  if (to.out == nullptr) return 0;
  if (to.w == nullptr || to.eps < 0.f || to.groups < 1 || d % to.groups != 0)
    return fail("%s: a norm over %d values in %d equal groups, with its weight and an eps", what, d, to.groups);
  return 0;
}

}  // namespace

#define HELD(shape, T, LAUNCH)                                                                                       \
  do {                                                                                                               \
    if ((shape).held == 0) LAUNCH(T, 0);                                                                             \
    else if ((shape).held == 1) LAUNCH(T, 1);                                                                        \
    else if ((shape).held == 2) LAUNCH(T, 2);                                                                        \
    else if ((shape).held == 4) LAUNCH(T, 4);                                                                        \
    else LAUNCH(T, 8);                                                                                               \
  } while (0)

// out: [n, d] in dtype (0 float32, 1 bfloat16), contiguous; x: float32, contiguous rows; w: float32 [d].
HFEE_API int hfee_group_norm(void* out, int dtype, const float* x, const int* rows, const float* w, float eps, int groups, int n,
                             int d, hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && d > 0 && x != nullptr && out != nullptr && out != (const void*)x, "group_norm: bad arguments");
  const NextNorm to{out, w, eps, groups};
  if (check_next(to, dtype, d, "group_norm")) return 1;
  if (n == 0) return 0;
  const RowShape s = row_shape(aligned(x, 16) && next_fits(to, d), d);
#define LAUNCH(T, K) group_norm_kernel<T, K><<<n, s.threads, norm_lds(s, to, d), stream>>>(x, rows, to, d)
  if (dtype == 0) HELD(s, float, LAUNCH); else HELD(s, bf16_t, LAUNCH);
#undef LAUNCH
  HFEE_CHECK_LAUNCH("group_norm");
  return 0;
}

// x, y, y2: float32 [n, d] contiguous; wy, wy2, w: float32 [d]; next (or null): [n, d] in dtype.
HFEE_API int hfee_pair_norm_add(float* x, const float* y, const float* y2, const float* wy, const float* wy2, float a, float b,
                                float eps, void* next, int dtype, const float* w, float next_eps, int groups, int n, int d,
                                hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && d > 0 && x != nullptr && y != nullptr && y2 != nullptr && wy != nullptr && wy2 != nullptr && eps >= 0.f,
               "pair_norm_add: bad arguments");
  const NextNorm to{next, w, next_eps, groups};
  if (check_next(to, dtype, d, "pair_norm_add")) return 1;
  if (n == 0) return 0;
  const RowShape s = row_shape(aligned(x, 16) && aligned(y, 16) && aligned(y2, 16) && aligned(wy, 16) && aligned(wy2, 16) && next_fits(to, d), d);
#define LAUNCH(T, K) pair_norm_add_kernel<T, K><<<n, s.threads, norm_lds(s, to, d), stream>>>(x, y, y2, wy, wy2, a, b, eps, to, d)
  if (dtype == 0) HELD(s, float, LAUNCH); else HELD(s, bf16_t, LAUNCH);
#undef LAUNCH
  HFEE_CHECK_LAUNCH("pair_norm_add");
  return 0;
}

// x, shared: float32 [n, d] contiguous; y: float32 [n * top, d], or [n, d] with summed; h and next in dtype.
HFEE_API int hfee_experts_join(float* x, const float* y, int summed, const int* chosen, const float* weights, int top, int experts,
                               const void* h, int64_t ldh, const float* shared, const float* gate, int64_t ldg, void* next,
                               int dtype, const float* w, float next_eps, int groups, int n, int d, hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && d > 0 && top >= 1 && experts >= 0 && x != nullptr && y != nullptr && chosen != nullptr && weights != nullptr &&
               h != nullptr && ldh >= d && ldg >= 0, "experts_join: bad arguments");
  const NextNorm to{next, w, next_eps, groups};
  if (check_next(to, dtype, d, "experts_join")) return 1;
  if (n == 0) return 0;
  const JoinArgs p{x, y, summed, chosen, weights, top, experts, h, ldh, shared, gate, ldg};
  const RowShape s = row_shape(aligned(x, 16) && aligned(y, 16) && aligned(shared, 16) && aligned(h, 16) && ldh % 4 == 0 && next_fits(to, d), d);
#define LAUNCH(T, K) experts_join_kernel<T, K><<<n, s.threads, norm_lds(s, to, d), stream>>>(p, to, d)
  if (dtype == 0) HELD(s, float, LAUNCH); else HELD(s, bf16_t, LAUNCH);
#undef LAUNCH
  HFEE_CHECK_LAUNCH("experts_join");
  return 0;
}

// out, z: [n, d] in dtype, rows ldo / ldz apart (out may be z); numbers: float32 [4].
HFEE_API int hfee_poly_norm(void* out, int64_t ldo, const void* z, int64_t ldz, int dtype, const float* numbers, float eps, int n,
                            int d, hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && d > 0 && out != nullptr && z != nullptr && numbers != nullptr && eps >= 0.f && ldo >= d && ldz >= d,
               "poly_norm: bad arguments");
  HFEE_REQUIRE(dtype == 0 || dtype == 1, "poly_norm: unknown dtype %d", dtype);
  if (n == 0) return 0;
  const RowShape s = row_shape(aligned(out, 16) && aligned(z, 16) && ldo % 4 == 0 && ldz % 4 == 0, d);
#define LAUNCH(T, K) poly_norm_kernel<T, K><<<n, s.threads, 0, stream>>>((T*)out, ldo, (const T*)z, ldz, numbers, eps, d)
  if (dtype == 0) HELD(s, float, LAUNCH); else HELD(s, bf16_t, LAUNCH);
#undef LAUNCH
  HFEE_CHECK_LAUNCH("poly_norm");
  return 0;
}
