// The gated delta rule with one decay a head and token:
//
//   S <- g_t S;  u_t = b_t (v_t - S^T k_t);  S <- S + k_t u_t^T;  o_t = S^T q_t
//
// delta_inputs: everything that enters it from a token's projections in one launch, in float32: the short convolutions
// with their SiLU, unit vectors a head for queries and keys (x / sqrt(sum x^2 + eps), queries also times a factor),
// decays exp(-exp(A_h) softplus(a + bias)) and writing strengths sigmoid(b); in a step of single tokens also the
// convolutions' state.
//
// delta_chunks: portions of many tokens in chunks of 64 on the float32 matrix instructions (recurrent.hip, rule 1, walks
// token by token).  With t and j counting from a chunk's first token, S the state that comes into the chunk, L its tokens,
// R(t, j) the product of the decays of the tokens behind j up to t, and G(t) that of all decays up to t:
//
//   u_t  = b_t (v_t - G(t) S^T k_t - sum_(j < t) R(t, j) (k_t . k_j) u_j)
//   o_t  = G(t) S^T q_t + sum_(j <= t) R(t, j) (q_t . k_j) u_j
//   S   <- G(L - 1) S + sum_j R(L - 1, j) k_j u_j^T
//
// The first line is a system with a unit lower triangle, (I + A) U = B - C S with rows b_t v_t of B and b_t G(t) k_t of C and
// A(t, j) = b_t R(t, j) (k_t . k_j) for j < t, so U = Y - W S with Y = (I + A)^-1 B and W = (I + A)^-1 C, which need no state:
//
//   delta_solve   a workgroup a (chunk, head), every chunk of every portion at once: the products of keys with keys and
//                 of queries with keys, the decays' products (each as a product of its own factors: no quotient, no
//                 logarithm, decays of 0 and 1 are as good as any), the triangle in blocks of 16 (the diagonal blocks
//                 inverted row by row, the rest by substitution), W, Y, P(t, j) = R(t, j) (q_t . k_j), G and R(L - 1, .);
//   delta_walk    a workgroup a (portion, head, 16 columns of S): from chunk to chunk, S in its waves' accumulators with a
//                 copy in LDS; a wave makes u and o of 16 of a chunk's tokens and the new S of its rows.  What a chunk
//                 needs of memory is asked for a chunk ahead.
//
// Operands and sums are float32 throughout.  Chunks count from the portion's first token, so how a prompt was cut moves
// the roundings and nothing else; a sum's order does not depend on what else the step holds.  Portions of fewer than
// kLeastTokens tokens are left to the kernel that walks token by token, whose layout of the state is kept.
#include "common.h"

using namespace hfee;

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

struct InputArgs {
  float* y;                    // [n, channels]: queries, keys, values
  int64_t ldy;
  float* decay;                // [n, heads]
  float* beta;                 // [n, heads]
  const void* x;               // [n, channels] projections in T
  int64_t ldx;
  const void* a;               // [n, heads] in T, ldx apart
  const void* b;
  void* state;                 // [slots][taps - 1][channels] in T, the newest last
  const float* taps;           // [channels][taps], the last column the current token's
  const float* dt_bias;
  const float* a_log;
  const int* token_segment;
  const int* segment_rows;
  const int* segment_slots;
  int n, channels, qk_width, dim, heads, keep;
  float unit_eps, q_factor;
};

// grid (groups of TT tokens, blocks of 256 fours of channels and one for decays and strengths).  A thread owns four
// channels and walks its tokens with the last inputs in registers; the dim / 4 threads of a head are neighbours in a wave
// (dim / 4 is a power of two up to 64) and meet over the sum of squares.
template <typename T, int K, int TT>
__global__ __launch_bounds__(256) void delta_inputs_kernel(InputArgs p) {
  const int t0 = blockIdx.x * TT, count = min(TT, p.n - t0);
  if (blockIdx.y == gridDim.y - 1) {
    for (int e = threadIdx.x; e < count * p.heads; e += blockDim.x) {
      const int t = t0 + e / p.heads, h = e % p.heads;
      const float za = to_float<T>(((const T*)p.a)[(int64_t)t * p.ldx + h]) + p.dt_bias[h];
      const float zb = to_float<T>(((const T*)p.b)[(int64_t)t * p.ldx + h]);
      p.decay[(int64_t)t * p.heads + h] = expf(-expf(p.a_log[h]) * softplus(za));
      p.beta[(int64_t)t * p.heads + h] = 1.0f / (1.0f + expf(-zb));
    }
    return;
  }
  const int c = (blockIdx.y * 256 + threadIdx.x) * 4;
  const bool mine = c < p.channels;
  const int cc = mine ? c : 0;
  const T* x = (const T*)p.x + cc;
  float now[TT][4], taps[K][4], past[K > 1 ? K - 1 : 1][4];
#pragma unroll
  for (int j = 0; j < TT; ++j) load4<T>(now[j], x + (int64_t)(t0 + (j < count ? j : 0)) * p.ldx);
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int k = 0; k < K; ++k) taps[k][i] = p.taps[(int64_t)(cc + i) * K + k];
  const int group = p.dim / 4;
  const bool unit = c < 2 * p.qk_width;
  const float factor = c < p.qk_width ? p.q_factor : 1.0f;
  int seg = -1;
  T* st = nullptr;
#pragma unroll
  for (int j = 0; j < TT; ++j) {
    if (j >= count) break;
    const int t = t0 + j;
    if (seg < 0 || t == p.segment_rows[p.token_segment[t]]) {      // (the tile's first token, or a portion's: what came before)
      seg = p.token_segment[t];
      const int at = t - p.segment_rows[seg];
      st = (T*)p.state + (int64_t)p.segment_slots[seg] * (K - 1) * p.channels + cc;
#pragma unroll
      for (int k = 0; k < K - 1; ++k) {        // past[k]: the input K - 1 - k tokens back
        const int back = K - 1 - k;
        load4<T>(past[k], at - back >= 0 ? x + (int64_t)(t - back) * p.ldx : st + (int64_t)(K - 1 + at - back) * p.channels);
      }
    }
    float y[4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float sum = 0.f;
#pragma unroll
      for (int k = 0; k < K - 1; ++k) sum = fmaf(taps[k][i], past[k][i], sum);
      sum = fmaf(taps[K - 1][i], now[j][i], sum);
      y[i] = mine ? sum / (1.0f + expf(-sum)) : 0.f;
      ss = fmaf(y[i], y[i], ss);
    }
    for (int off = group >> 1; off > 0; off >>= 1) ss += __shfl_xor(ss, off, kWave);
    if (unit) {
      const float inv = factor / sqrtf(ss + p.unit_eps);
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] *= inv;
    }
    if (mine) store4<float>(p.y + (int64_t)t * p.ldy + c, y);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int k = 0; k + 1 < K - 1; ++k) past[k][i] = past[k + 1][i];
      if (K > 1) past[K > 1 ? K - 2 : 0][i] = now[j][i];
    }
    if (p.keep && mine) {                      // (every token is its portion's only one: the thread's own channels)
#pragma unroll
      for (int k = 0; k < K - 1; ++k) store4<T>(st + (int64_t)k * p.channels, past[k]);
    }
  }
}

constexpr int kChunk = 64, kLeastTokens = 16, kColumns = 16, kPitch = kChunk + 4;

struct DeltaArgs {
  float* out;
  int64_t ldo;
  float* state;
  const float* q;
  int64_t ldq;
  const float* k;
  int64_t ldk;
  const float* v;
  int64_t ldv;
  const float* decay;
  int64_t ldd;
  const float* beta;
  int64_t ldb;
  float* P;                  // [heads][rows of the step][kChunk]
  float* W;                  // [heads][rows][D]
  float* Y;                  // [heads][rows][V]
  float* upto;               // [heads][rows]: G(t)
  float* behind;             // [heads][rows]: R(L - 1, t)
  const int* segment_rows;
  const int* segment_lengths;
  const int* segment_slots;
  int rows, heads, qk_heads, D, V, rows_a_lane;
};

// A 16 x 16 x 4 instruction: lane (r, g) = (lane % 16, lane / 16) holds row (or column) r of its operand for the label g,
// and ends with rows 4 g + i of column r.  Label g of instruction i stands for element 4 g + i of a step of 16, so an
// operand that lies in rows is a load of four neighbours, and what one product leaves in the registers is the column
// operand of the next.
__device__ __forceinline__ f32x4 block_product(f32x4 rows, f32x4 columns, f32x4 acc) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(rows[i], columns[i], acc, 0, 0, 0);
  return acc;
}

template <int DT>
__global__ __launch_bounds__(256) void delta_solve_kernel(DeltaArgs p) {
  __shared__ float beta[kChunk], upto[kChunk];
  __shared__ __attribute__((aligned(16))) float R[kChunk * kPitch], A[kChunk * kPitch], T[kChunk * 20];
  const int seg = blockIdx.z, h = blockIdx.y, len = p.segment_lengths[seg], first = blockIdx.x * kChunk;
  if (len < kLeastTokens || first >= len) return;
  const int row0 = p.segment_rows[seg] + first, L = min(kChunk, len - first);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int kg = h / (p.heads / p.qk_heads);
  const int64_t at = (int64_t)h * p.rows + row0;
  const float* kb = p.k + (int64_t)row0 * p.ldk + (int64_t)kg * p.D;
  const float* qb = p.q + (int64_t)row0 * p.ldq + (int64_t)kg * p.D;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};

  if (wave == 0) {           // tokens behind the chunk's last: a decay of one, a strength of zero
    const float decay = lane < L ? p.decay[(int64_t)(row0 + lane) * p.ldd + h] : 1.0f;
    beta[lane] = lane < L ? p.beta[(int64_t)(row0 + lane) * p.ldb + h] : 0.f;
    float product = 1.0f, all = 1.0f, mine = 1.0f, last = 1.0f;
#pragma unroll 8
    for (int t = 0; t < kChunk; ++t) {
      const float d = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(decay), t));
      all *= d;
      product = t > lane ? product * d : 1.0f;
      R[t * kPitch + lane] = product;
      if (t == lane) mine = all;
      if (t == L - 1) last = product;
    }
    upto[lane] = mine;
    if (lane < L) {
      p.upto[at + lane] = mine;
      p.behind[at + lane] = last;
    }
  }

  // waves 0, 1: keys with keys; 2, 3: queries with keys; of the four row blocks two a wave, five tiles in all
  const float* own = wave < 2 ? kb : qb;
  const int64_t ld_own = wave < 2 ? p.ldk : p.ldq;
  const int high = 3 - (wave & 1), low = wave & 1;
  f32x4 tiles[5];
  auto rows_of = [&](const float* base, int64_t ld, int block, f32x4 (&o)[DT]) {
    const float* row = base + (int64_t)min(block * 16 + r, L - 1) * ld;
#pragma unroll
    for (int s = 0; s < DT; ++s) {
      const int d = s * 16 + 4 * g;
      o[s] = *reinterpret_cast<const f32x4*>(row + (d < p.D ? d : 0));
      if (d >= p.D) o[s] = zero;
    }
  };
  {
    f32x4 mine[DT], keys[DT];
    int block = high;
    rows_of(own, ld_own, block, mine);
#pragma unroll
    for (int i = 0; i < 5; ++i) {
      if (i == high + 1) {
        block = low;
        rows_of(own, ld_own, block, mine);
      }
      rows_of(kb, p.ldk, i <= high ? i : i - high - 1, keys);
      f32x4 acc = zero, acc2 = zero;
#pragma unroll
      for (int s = 0; s < DT; s += 2) {
        acc = block_product(mine[s], keys[s], acc);
        if (s + 1 < DT) acc2 = block_product(mine[s + 1], keys[s + 1], acc2);
      }
      tiles[i] = acc + acc2;
    }
  }
  __syncthreads();           // R and the strengths are there
#pragma unroll
  for (int i = 0; i < 5; ++i) {
    const int block = i <= high ? high : low, j = (i <= high ? i : i - high - 1) * 16 + r;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = block * 16 + 4 * g + e;
      const float x = tiles[i][e] * R[t * kPitch + j];
      if (wave < 2) A[t * kPitch + j] = j < t ? -beta[t] * x : 0.f;      // (-A)
      else if (t < L) p.P[(at + t) * kChunk + j] = j <= t ? x : 0.f;
    }
  }
  __syncthreads();
  {                          // (I + A)^-1 of a diagonal block, a lane a column (the four g alike)
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float sum = i == r ? 1.0f : 0.f;
      const float* row = &A[(wave * 16 + i) * kPitch + wave * 16];
#pragma unroll
      for (int j = 0; j < i; ++j) sum = fmaf(row[j], x[j], sum);
      x[i] = sum;
      if (g == 0) T[(wave * 16 + i) * 20 + r] = sum;
    }
  }
  __syncthreads();
  f32x4 inverse[4], below[6];
#pragma unroll
  for (int I = 0; I < 4; ++I) {
    inverse[I] = *reinterpret_cast<const f32x4*>(&T[(I * 16 + r) * 20 + 4 * g]);
#pragma unroll
    for (int J = 0; J < I; ++J)
      below[I * (I - 1) / 2 + J] = *reinterpret_cast<const f32x4*>(&A[(I * 16 + r) * kPitch + J * 16 + 4 * g]);
  }
  const int key_tiles = (p.D + 15) / 16, value_tiles = (p.V + 15) / 16;
  const float* vb = p.v + (int64_t)row0 * p.ldv + (int64_t)h * p.V;
  for (int tile = wave; tile < key_tiles + value_tiles; tile += 4) {
    const bool keys = tile < key_tiles;
    const int col = (keys ? tile : tile - key_tiles) * 16 + r, width = keys ? p.D : p.V;
    const bool live = col < width;
    const float* base = (keys ? kb : vb) + (live ? col : 0);
    const int64_t ld = keys ? p.ldk : p.ldv;
    f32x4 x[4];
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int e = 0; e < 4; ++e) x[I][e] = base[(int64_t)min(I * 16 + 4 * g + e, L - 1) * ld];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = I * 16 + 4 * g + e;
        x[I][e] *= keys ? beta[t] * upto[t] : beta[t];
      }
#pragma unroll
      for (int J = 0; J < I; ++J) x[I] = block_product(below[I * (I - 1) / 2 + J], x[J], x[I]);
      x[I] = block_product(inverse[I], x[I], zero);
    }
    float* to = (keys ? p.W : p.Y) + at * width + col;
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = I * 16 + 4 * g + e;
        if (live && t < L) to[(int64_t)t * width] = x[I][e];
      }
  }
}

// What a lane of the walk needs of a chunk.
template <int DT>
struct WalkOperands {
  static constexpr int TILES = (DT + 3) / 4;      // groups of 16 rows of S a wave owns
  f32x4 q[DT], w[DT];                             // its token's query and row of W, as the row operands
  f32x4 s[4];                                     // its token's row of P
  float y[4], upto[4], behind[4];                 // of tokens 4 g + i of the wave's 16, in its column
  float k[TILES][16];                             // the chunk's keys in its rows of S
  float all;                                      // G(L - 1)
};

// DT: the key size in groups of 16, filled up (dims at and beyond D count as zeros).
template <int DT>
__global__ __launch_bounds__(256) void delta_walk_kernel(DeltaArgs p) {
  typedef WalkOperands<DT> Operands;
  constexpr int TILES = Operands::TILES, PITCH = DT * 16 + 4;
  __shared__ __attribute__((aligned(16))) float St[kColumns * PITCH];      // S transposed: [column][row]
  __shared__ __attribute__((aligned(16))) float Ut[kColumns * kPitch];     // u: [column][token]
  __shared__ __attribute__((aligned(16))) float Ub[kColumns * kPitch];     // u times R(L - 1, token)
  const int seg = blockIdx.z, h = blockIdx.x, len = p.segment_lengths[seg];
  if (len < kLeastTokens) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int col = blockIdx.y * kColumns + r;
  const bool live = col < p.V;
  const int row_first = p.segment_rows[seg], kg = h / (p.heads / p.qk_heads);
  const int blocks = (p.V + 3) / 4, per = p.rows_a_lane;
  float* head_state = p.state + ((int64_t)p.segment_slots[seg] * p.heads + h) * blocks * (per * 64);
  auto place = [&](int d) { return (int64_t)(col >> 2) * (per * 64) + (d % per) * 64 + (col & 3) * 16 + d / per; };
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};

  f32x4 S[TILES];
#pragma unroll
  for (int tile = 0; tile < TILES; ++tile) {
    const int d0 = (wave + 4 * tile) * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i) S[tile][i] = live && d0 + i < p.D ? head_state[place(d0 + i)] : 0.f;
  }

  // Every load is made, with a place inside the portion and the head for what lies outside of either (a load behind
  // a condition would be waited for where it stands): what must not count meets a zero where it is used.
  const int first_four = 4 * g < p.D ? 4 * g : 0;
  auto load = [&](int first, Operands& o) {
    const int L = min(kChunk, len - first);
    const int64_t row0 = row_first + first, at = (int64_t)h * p.rows + row0;
    const float* qb = p.q + row0 * p.ldq + (int64_t)kg * p.D;
    const float* kb = p.k + row0 * p.ldk + (int64_t)kg * p.D;
    const float* wb = p.W + at * p.D;
    const int t = min(wave * 16 + r, L - 1), ldq = (int)p.ldq, ldk = (int)p.ldk;
#pragma unroll
    for (int s = 0; s < DT; ++s) {
      const int d = s * 16 + 4 * g < p.D ? s * 16 + 4 * g : first_four;
      o.w[s] = *reinterpret_cast<const f32x4*>(wb + t * p.D + d);
      o.q[s] = *reinterpret_cast<const f32x4*>(qb + t * ldq + d);
    }
#pragma unroll
    for (int s = 0; s < 4; ++s) o.s[s] = *reinterpret_cast<const f32x4*>(p.P + (at + t) * kChunk + s * 16 + 4 * g);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = min(wave * 16 + 4 * g + i, L - 1);
      o.y[i] = p.Y[(at + row) * p.V + (live ? col : 0)];
      o.upto[i] = p.upto[at + row];
      o.behind[i] = p.behind[at + row];
    }
    o.all = p.upto[at + L - 1];
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int row = min((e >> 2) * 16 + 4 * g + (e & 3), L - 1);
#pragma unroll
      for (int tile = 0; tile < TILES; ++tile) {
        const int d = (wave + 4 * tile) * 16 + r;
        o.k[tile][e] = kb[row * ldk + (d < p.D ? d : 0)];
      }
    }
  };
  auto copy_state = [&]() {      // (rows at and beyond D, where the operands hold other numbers, are zeros)
#pragma unroll
    for (int tile = 0; tile < TILES; ++tile) {
      const int d0 = (wave + 4 * tile) * 16 + 4 * g;
      if (wave + 4 * tile < DT) *reinterpret_cast<f32x4*>(&St[r * PITCH + d0]) = d0 < p.D ? S[tile] : zero;
    }
  };

  auto step = [&](int first, Operands& now, Operands& next) {
    const int L = min(kChunk, len - first);
    load(first + kChunk < len ? first + kChunk : first, next);
    // u = Y - W S and G q S: the lane ends with tokens wave * 16 + 4 g + i of its column
    f32x4 u0 = zero, u1 = zero, o0 = zero, o1 = zero;
#pragma unroll
    for (int s = 0; s < DT; ++s) {
      const f32x4 st = *reinterpret_cast<const f32x4*>(&St[r * PITCH + s * 16 + 4 * g]);
      if (s & 1) {
        u1 = block_product(now.w[s], st, u1);
        o1 = block_product(now.q[s], st, o1);
      } else {
        u0 = block_product(now.w[s], st, u0);
        o0 = block_product(now.q[s], st, o0);
      }
    }
    f32x4 u, ub;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool in = wave * 16 + 4 * g + i < L;
      u[i] = in ? now.y[i] - (u0[i] + u1[i]) : 0.f;
      ub[i] = u[i] * now.behind[i];
      o0[i] = (o0[i] + o1[i]) * now.upto[i];
    }
    *reinterpret_cast<f32x4*>(&Ut[r * kPitch + wave * 16 + 4 * g]) = u;
    *reinterpret_cast<f32x4*>(&Ub[r * kPitch + wave * 16 + 4 * g]) = ub;
    __syncthreads();             // every wave has read the copy of the old S, and all u are there
#pragma unroll
    for (int tile = 0; tile < TILES; ++tile) S[tile] = S[tile] * now.all;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const f32x4 ubs = *reinterpret_cast<const f32x4*>(&Ub[r * kPitch + s * 16 + 4 * g]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int tile = 0; tile < TILES; ++tile)
          S[tile] = __builtin_amdgcn_mfma_f32_16x16x4f32(now.k[tile][s * 4 + i], ubs[i], S[tile], 0, 0, 0);
    }
    copy_state();
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      if (s > wave) break;       // (later tokens do not count)
      o0 = block_product(now.s[s], *reinterpret_cast<const f32x4*>(&Ut[r * kPitch + s * 16 + 4 * g]), o0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = wave * 16 + 4 * g + i;
      if (live && t < L) p.out[(int64_t)(row_first + first + t) * p.ldo + (int64_t)h * p.V + col] = o0[i];
    }
    __syncthreads();             // the new copy of S is there, and every wave has read the u
  };
  Operands even, odd;            // (by turns: copying one into the other would wait for the loads)
  load(0, even);
  copy_state();
  __syncthreads();
  for (int first = 0; first < len; first += 2 * kChunk) {
    step(first, even, odd);
    if (first + kChunk >= len) break;
    step(first + kChunk, odd, even);
  }
#pragma unroll
  for (int tile = 0; tile < TILES; ++tile) {
    const int d0 = (wave + 4 * tile) * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (live && d0 + i < p.D) head_state[place(d0 + i)] = S[tile][i];
  }
}

bool power_of_two(int v) { return v > 0 && (v & (v - 1)) == 0; }

}  // namespace

// Whether hfee_delta_inputs takes these sizes.
HFEE_API int hfee_delta_inputs_fit(int channels, int dim, int taps) {
  return channels % 4 == 0 && dim % 4 == 0 && power_of_two(dim / 4) && dim <= 256 && taps >= 1 && taps <= 4;
}

// x: [n, channels] in dtype (0 float32, 1 bfloat16), the first qk_width columns queries, the next qk_width keys (heads of
// dim), the rest values; a, b: [n, heads] like x, rows ldx apart; y: float32 [n, channels]; decay, beta: float32
// [n, heads] contiguous.  keep: every token is its segment's only one, and the state gets its input.
HFEE_API int hfee_delta_inputs(float* y, int64_t ldy, float* decay, float* beta, const void* x, int64_t ldx, const void* a,
                               const void* b, int dtype, void* state, const float* taps, int taps_count, const float* dt_bias,
                               const float* a_log, const int* token_segment, const int* segment_rows, const int* segment_slots,
                               int n, int channels, int qk_width, int dim, int heads, float unit_eps, float q_factor, int keep,
                               hipStream_t stream) {
  HFEE_REQUIRE(n >= 0 && heads > 0 && qk_width > 0 && 2 * qk_width <= channels && dim > 0 && qk_width % dim == 0, "delta_inputs: bad sizes");
  HFEE_REQUIRE(hfee_delta_inputs_fit(channels, dim, taps_count), "delta_inputs: %d channels in heads of %d with %d taps", channels, dim, taps_count);
  HFEE_REQUIRE(dtype == 0 || dtype == 1, "delta_inputs: unknown dtype %d", dtype);
  HFEE_REQUIRE(ldx % 4 == 0 && ldx >= channels && ldy % 4 == 0 && ldy >= channels &&
               (((uintptr_t)y | (uintptr_t)x | (uintptr_t)state) & 15) == 0, "delta_inputs: rows must be aligned");
  if (n == 0) return 0;
  const InputArgs p{y, ldy, decay, beta, x, ldx, a, b, state, taps, dt_bias, a_log, token_segment, segment_rows, segment_slots,
                    n, channels, qk_width, dim, heads, keep, unit_eps, q_factor};
  const int columns = (channels / 4 + 255) / 256 + 1;
  HFEE_REQUIRE(columns <= 65535, "delta_inputs: too many channels");
  const bool few = n <= 64;
#define LAUNCH(T, K)                                                                                                 \
  do {                                                                                                               \
    if (few) delta_inputs_kernel<T, K, 1><<<dim3(n, columns), 256, 0, stream>>>(p);                                  \
    else delta_inputs_kernel<T, K, 8><<<dim3((n + 7) / 8, columns), 256, 0, stream>>>(p);                            \
  } while (0)
#define PICK(T)                                                                                                      \
  if (taps_count == 1) LAUNCH(T, 1); else if (taps_count == 2) LAUNCH(T, 2); else if (taps_count == 3) LAUNCH(T, 3); \
  else LAUNCH(T, 4)
  if (dtype == 0) { PICK(float); } else { PICK(bf16_t); }
#undef PICK
#undef LAUNCH
  HFEE_CHECK_LAUNCH("delta_inputs");
  return 0;
}

HFEE_API int hfee_delta_chunks_least() { return kLeastTokens; }

// Portions of at least hfee_delta_chunks_least() tokens; the others are left alone.  longest: the step's longest portion;
// rows: the step's rows; scratch: float32 [heads * rows * (64 + dim + vdim + 2)], 16-byte aligned.  dim a multiple of 4, at
// most 256; q and k rows a multiple of four floats apart, 16-byte aligned.
HFEE_API int hfee_delta_chunks(float* out, int64_t ldo, float* state, const float* q, int64_t ldq, const float* k, int64_t ldk,
                               const float* v, int64_t ldv, const float* decay, int64_t ldd, const float* beta, int64_t ldb,
                               const int* segment_rows, const int* segment_lengths, const int* segment_slots, int segments,
                               int longest, int rows, int heads, int qk_heads, int dim, int vdim, int rows_a_lane, float* scratch,
                               int64_t scratch_floats, hipStream_t stream) {
  HFEE_REQUIRE(segments >= 0 && segments <= 65535 && rows >= 0, "delta_chunks: bad segment count");
  if (segments == 0 || longest < kLeastTokens) return 0;
  HFEE_REQUIRE(heads > 0 && qk_heads > 0 && heads % qk_heads == 0 && heads <= 65535,
               "delta_chunks: %d heads are not a multiple of %d query/key heads", heads, qk_heads);
  HFEE_REQUIRE(dim >= 4 && dim <= 256 && dim % 4 == 0 && vdim >= 1 && rows_a_lane >= 1 && 16 * rows_a_lane >= dim,
               "delta_chunks: key sizes of 4 to 256 in fours");
  HFEE_REQUIRE(ldq % 4 == 0 && ldk % 4 == 0 && (((uintptr_t)q | (uintptr_t)k | (uintptr_t)scratch) & 15) == 0,
               "delta_chunks: query and key rows must be 16-byte aligned");
  HFEE_REQUIRE(ldq >= (int64_t)qk_heads * dim && ldk >= (int64_t)qk_heads * dim && ldv >= (int64_t)heads * vdim &&
               ldo >= (int64_t)heads * vdim && ldd >= heads && ldb >= heads && ldq < (1 << 24) && ldk < (1 << 24), "delta_chunks: rows too short");
  const int64_t places = (int64_t)heads * rows;
  HFEE_REQUIRE(longest <= rows && scratch != nullptr && scratch_floats >= places * (kChunk + dim + vdim + 2),
               "delta_chunks: the scratch needs room for every row of every head");
  HFEE_REQUIRE((vdim + kColumns - 1) / kColumns <= 65535, "delta_chunks: values too wide");
  float* P = scratch;
  float* W = P + places * kChunk;
  float* upto = W + places * dim;
  float* behind = upto + places;
  float* Y = behind + places;
  const DeltaArgs p{out, ldo, state, q, ldq, k, ldk, v, ldv, decay, ldd, beta, ldb, P, W, Y, upto, behind, segment_rows,
                    segment_lengths, segment_slots, rows, heads, qk_heads, dim, vdim, rows_a_lane};
  const dim3 solve((longest + kChunk - 1) / kChunk, heads, segments), walk(heads, (vdim + kColumns - 1) / kColumns, segments);
#define LAUNCH(DT)                                                                                                   \
  do {                                                                                                               \
    delta_solve_kernel<DT><<<solve, 256, 0, stream>>>(p);                                                            \
    HFEE_CHECK_LAUNCH("delta_chunks (solve)");                                                                       \
    delta_walk_kernel<DT><<<walk, 256, 0, stream>>>(p);                                                              \
  } while (0)
  if (dim <= 32) LAUNCH(2); else if (dim <= 64) LAUNCH(4); else if (dim <= 128) LAUNCH(8); else LAUNCH(16);
#undef LAUNCH
  HFEE_CHECK_LAUNCH("delta_chunks (walk)");
  return 0;
}
