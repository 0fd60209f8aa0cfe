// Linear attention with one fixed decay a head, for portions of many tokens: the recurrence of recurrent.hip
// (rule 0, S <- a S + k_t v_t^T, o_t = S^T q_t) in chunks of 64 tokens on the float32 matrix instructions.
//
// With t and j counting from a chunk's first token, S the state that comes into the chunk and L its tokens:
//
//   o_t  = a^(t+1) q_t S + sum_(j <= t) a^(t-j) (q_t . k_j) v_j
//   S   <- a^L S + sum_j a^(L-1-j) k_j v_j^T
//
// No power of a is ever negative, so any decay from 0 to 1 is safe.  Two kernels:
//
//   chunk_scores  P[t][j] = a^(t-j) (q_t . k_j) for j <= t, 0 behind it: a workgroup a (chunk, head), every chunk of
//                 every portion at once; a wave one of the four 32 x 32 tiles;
//   chunk_walk    a workgroup a (portion, head, 16 columns of S): from chunk to chunk, S in its waves' accumulators
//                 (a wave owns every fourth group of 16 rows) with a copy in LDS that the products q S read; a wave
//                 makes the outputs of 16 of a chunk's tokens.  What a chunk needs of memory is asked for a chunk
//                 ahead and goes from memory into the operands' registers: an element is used once a workgroup.
//
// Operands and sums are float32 throughout.  Chunks count from the portion's first token, so how a prompt was cut
// moves the roundings and nothing else; a sum's order does not depend on what else the step holds.  Portions of
// fewer than kLeastTokens tokens are left to the kernel that walks token by token.
//
// The state lies as that kernel keeps it: of a head in blocks of four columns, [block][i][column][part], row
// d = rows_a_lane * part + i.
#include "common.h"

using namespace hfee;

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int kChunk = 64, kLeastTokens = 16, kColumns = 16;

struct ChunkArgs {
  float* out;
  int64_t ldo;
  float* state;
  const float* q;
  int64_t ldq;
  const float* k;
  int64_t ldk;
  const float* v;
  int64_t ldv;
  const float* decay;        // [heads]
  float* scores;             // [heads][rows of the step][kChunk]
  const int* segment_rows;
  const int* segment_lengths;
  const int* segment_slots;
  int rows, heads, qk_heads, D, V, rows_a_lane;
};

// powers[i] = a^i, i = 0 .. kChunk (0^0 = 1)
__device__ __forceinline__ void make_powers(float* powers, float a) {
  if (threadIdx.x <= kChunk) powers[threadIdx.x] = threadIdx.x == 0 ? 1.0f : powf(a, (float)threadIdx.x);
}

// register r of a lane in a 32 x 32 tile: row 8 (r / 4) + 4 (lane / 32) + r % 4, column lane % 32.  The k index of a
// matrix instruction is a label that both operands share: label (step s, half of the lanes, i) means dim
// 8 s + 4 half + i, so that a lane's operands of four instructions are sixteen neighbouring bytes.
__global__ __launch_bounds__(256) void chunk_scores_kernel(ChunkArgs p) {
  __shared__ float powers[kChunk + 1];
  const int seg = blockIdx.z, h = blockIdx.y, len = p.segment_lengths[seg], first = blockIdx.x * kChunk;
  if (len < kLeastTokens || first >= len) return;
  make_powers(powers, p.decay[h]);
  __syncthreads();
  const int row0 = p.segment_rows[seg] + first, L = min(kChunk, len - first);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 31, half = lane >> 5;
  const int t0 = (wave >> 1) * 32, j0 = (wave & 1) * 32;
  float* scores = p.scores + ((int64_t)h * p.rows + row0) * kChunk;
  f32x16 acc;
#pragma unroll
  for (int r = 0; r < 16; ++r) acc[r] = 0.f;
  if (j0 <= t0 && t0 < L) {
    const int g = h / (p.heads / p.qk_heads);
    const float* qr = p.q + (int64_t)(row0 + min(t0 + col, L - 1)) * p.ldq + (int64_t)g * p.D + half * 4;
    const float* kr = p.k + (int64_t)(row0 + min(j0 + col, L - 1)) * p.ldk + (int64_t)g * p.D + half * 4;
    for (int d0 = 0; d0 < p.D; d0 += 32) {          // (four steps' operands on their way at a time)
      f32x4 a[4], b[4];
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const int d = d0 + 8 * s;
        a[s] = b[s] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (d + half * 4 < p.D) {
          a[s] = *reinterpret_cast<const f32x4*>(qr + d);
          b[s] = *reinterpret_cast<const f32x4*>(kr + d);
        }
      }
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(a[s][i], b[s][i], acc, 0, 0, 0);
    }
  }
  const int j = j0 + col;
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int t = t0 + 8 * (r >> 2) + 4 * half + (r & 3);
    if (t < L) scores[(int64_t)t * kChunk + j] = j <= t ? acc[r] * powers[t - j] : 0.f;
  }
}

// What a lane of the walk needs of a chunk.  A 16 x 16 x 4 instruction: lane (r, g) = (lane % 16, lane / 16) holds
// row (or column) r of its operand for the label g; the four instructions of a step of 16 take label (g, i) for
// element 16 step + 4 g + i.
template <int DT>
struct ChunkOperands {
  static constexpr int TILES = (DT + 3) / 4;      // groups of 16 rows of S a wave owns
  f32x4 q[DT];                                    // its token's query, as the row operand of q S
  f32x4 s[4];                                     // its token's scores, as the row operand of P v
  float v[16];                                    // the chunk's values in its column
  float k[TILES][16];                             // the chunk's keys in its rows of S
};

// DT: the key size in groups of 16, filled up (dims at and beyond D count as zeros).
template <int DT>
__global__ __launch_bounds__(256) void chunk_walk_kernel(ChunkArgs p) {
  typedef ChunkOperands<DT> Operands;
  constexpr int TILES = Operands::TILES, PITCH = DT * 16 + 4;
  __shared__ float powers[kChunk + 1];
  __shared__ __attribute__((aligned(16))) float St[kColumns * PITCH];      // S transposed: [column][row]
  // (heads first: with a multiple of eight heads a head's workgroups, which read the same queries and keys, run on
  // one of the eight dies)
  const int seg = blockIdx.z, h = blockIdx.x, len = p.segment_lengths[seg];
  if (len < kLeastTokens) return;
  make_powers(powers, p.decay[h]);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int col = blockIdx.y * kColumns + r;
  const bool live = col < p.V;
  const int row_first = p.segment_rows[seg], kg = h / (p.heads / p.qk_heads);
  const int blocks = (p.V + 3) / 4, R = p.rows_a_lane;
  float* head_state = p.state + ((int64_t)p.segment_slots[seg] * p.heads + h) * blocks * (R * 64);
  auto place = [&](int d) { return (int64_t)(col >> 2) * (R * 64) + (d % R) * 64 + (col & 3) * 16 + d / R; };

  f32x4 S[TILES];
#pragma unroll
  for (int tile = 0; tile < TILES; ++tile) {
    const int d0 = (wave + 4 * tile) * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i) S[tile][i] = live && d0 + i < p.D ? head_state[place(d0 + i)] : 0.f;
  }

  // Every load is made, with a place inside the portion and the head for what lies outside of either (a load behind
  // a condition would be waited for where it stands): what must not count meets a zero where it is used.
  const int q_step = 4 * g < p.D ? 4 * g : 0;
  auto load = [&](int first, Operands& o) {
    const int L = min(kChunk, len - first);
    const int64_t row0 = row_first + first;
    const float* qb = p.q + row0 * p.ldq + (int64_t)kg * p.D;
    const float* kb = p.k + row0 * p.ldk + (int64_t)kg * p.D;
    const float* vb = p.v + row0 * p.ldv + (int64_t)h * p.V;
    const float* sb = p.scores + ((int64_t)h * p.rows + row0) * kChunk;
    const int t = min(wave * 16 + r, L - 1), ldq = (int)p.ldq, ldk = (int)p.ldk, ldv = (int)p.ldv;
#pragma unroll
    for (int s = 0; s < DT; ++s) o.q[s] = *reinterpret_cast<const f32x4*>(qb + t * ldq + (s * 16 + 4 * g < p.D ? s * 16 + 4 * g : q_step));
#pragma unroll
    for (int s = 0; s < 4; ++s) o.s[s] = *reinterpret_cast<const f32x4*>(sb + t * kChunk + s * 16 + 4 * g);
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int row = min((e >> 2) * 16 + 4 * g + (e & 3), L - 1);
      o.v[e] = vb[row * ldv + (live ? col : 0)];
#pragma unroll
      for (int tile = 0; tile < TILES; ++tile) {
        const int d = (wave + 4 * tile) * 16 + r;
        o.k[tile][e] = kb[row * ldk + (d < p.D ? d : 0)];
      }
    }
  };
  auto copy_state = [&]() {      // (rows at and beyond D, where the queries hold other numbers, are zeros)
#pragma unroll
    for (int tile = 0; tile < TILES; ++tile) {
      const int d0 = (wave + 4 * tile) * 16 + 4 * g;
      if (wave + 4 * tile < DT) *reinterpret_cast<f32x4*>(&St[r * PITCH + d0]) = d0 < p.D ? S[tile] : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  };

  auto step = [&](int first, Operands& now, Operands& next) {
    const int L = min(kChunk, len - first);
    load(first + kChunk < len ? first + kChunk : first, next);
    // o = a^(t+1) q S + P v: the lane ends with tokens wave * 16 + 4 g + i of its column
    f32x4 o0 = {0.f, 0.f, 0.f, 0.f}, o1 = o0;
#pragma unroll
    for (int s = 0; s < DT; ++s) {
      const f32x4 st = *reinterpret_cast<const f32x4*>(&St[r * PITCH + s * 16 + 4 * g]);
#pragma unroll
      for (int i = 0; i < 4; i += 2) {
        o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(now.q[s][i], st[i], o0, 0, 0, 0);
        o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(now.q[s][i + 1], st[i + 1], o1, 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) o0[i] = (o0[i] + o1[i]) * powers[wave * 16 + 4 * g + i + 1];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      if (s > wave) break;                                // (the scores of later tokens are zeros)
#pragma unroll
      for (int i = 0; i < 4; ++i) o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(now.s[s][i], now.v[s * 4 + i], o0, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = wave * 16 + 4 * g + i;
      if (live && t < L) p.out[(int64_t)(row_first + first + t) * p.ldo + (int64_t)h * p.V + col] = o0[i];
    }
    // S <- a^L S + sum_j a^(L-1-j) k_j v_j^T
    const float all = powers[L];
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int j = (e >> 2) * 16 + 4 * g + (e & 3);
      now.v[e] *= j < L ? powers[L - 1 - j] : 0.f;
    }
#pragma unroll
    for (int tile = 0; tile < TILES; ++tile) S[tile] = S[tile] * all;
#pragma unroll
    for (int e = 0; e < 16; ++e)
#pragma unroll
      for (int tile = 0; tile < TILES; ++tile)
        S[tile] = __builtin_amdgcn_mfma_f32_16x16x4f32(now.k[tile][e], now.v[e], S[tile], 0, 0, 0);
    __syncthreads();                                      // every wave has read the copy of the old S
    copy_state();
    __syncthreads();
  };
  Operands even, odd;      // (by turns: copying one into the other would wait for the loads)
  load(0, even);
  copy_state();
  __syncthreads();                                        // the powers and the copy of S are there
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

}  // namespace

HFEE_API int hfee_linear_chunks_least() { return kLeastTokens; }

// Portions of at least hfee_linear_chunks_least() tokens; the others are left alone.  longest: the step's longest
// portion.  scores: float32 [heads * rows * 64]; rows: the step's rows.  dim a multiple of 4, at most 256; q and k
// rows a multiple of four floats apart, 16-byte aligned.
HFEE_API int hfee_linear_chunks(float* out, int64_t ldo, float* state, const float* q, int64_t ldq, const float* k, int64_t ldk,
                                const float* v, int64_t ldv, const float* decay, const int* segment_rows,
                                const int* segment_lengths, const int* segment_slots, int segments, int longest, int rows,
                                int heads, int qk_heads, int dim, int vdim, int rows_a_lane, float* scores,
                                int64_t score_floats, hipStream_t stream) {
  HFEE_REQUIRE(segments >= 0 && segments <= 65535 && rows >= 0, "linear_chunks: bad segment count");
  if (segments == 0 || longest < kLeastTokens) return 0;
  HFEE_REQUIRE(heads > 0 && qk_heads > 0 && heads % qk_heads == 0 && heads <= 65535,
               "linear_chunks: %d heads are not a multiple of %d query/key heads", heads, qk_heads);
  HFEE_REQUIRE(dim >= 4 && dim <= 256 && dim % 4 == 0 && vdim >= 1 && rows_a_lane >= 1 && 16 * rows_a_lane >= dim,
               "linear_chunks: key sizes of 4 to 256 in fours");
  HFEE_REQUIRE(ldq % 4 == 0 && ldk % 4 == 0 && (((uintptr_t)q | (uintptr_t)k | (uintptr_t)scores) & 15) == 0,
               "linear_chunks: query and key rows must be 16-byte aligned");
  HFEE_REQUIRE(ldq >= (int64_t)qk_heads * dim && ldk >= (int64_t)qk_heads * dim && ldv >= (int64_t)heads * vdim &&
               ldo >= (int64_t)heads * vdim, "linear_chunks: rows too short");
  HFEE_REQUIRE(longest <= rows && scores != nullptr && score_floats >= (int64_t)heads * rows * kChunk,
               "linear_chunks: the scores need room for every row of every head");
  const ChunkArgs p{out, ldo, state, q, ldq, k, ldk, v, ldv, decay, scores, segment_rows, segment_lengths, segment_slots,
                    rows, heads, qk_heads, dim, vdim, rows_a_lane};
  const int chunks = (longest + kChunk - 1) / kChunk;
  chunk_scores_kernel<<<dim3(chunks, heads, segments), 256, 0, stream>>>(p);
  HFEE_CHECK_LAUNCH("linear_chunks (scores)");
  HFEE_REQUIRE((vdim + kColumns - 1) / kColumns <= 65535, "linear_chunks: values too wide");
  const dim3 grid(heads, (vdim + kColumns - 1) / kColumns, segments);
  if (dim <= 32) chunk_walk_kernel<2><<<grid, 256, 0, stream>>>(p);
  else if (dim <= 64) chunk_walk_kernel<4><<<grid, 256, 0, stream>>>(p);
  else if (dim <= 128) chunk_walk_kernel<8><<<grid, 256, 0, stream>>>(p);
  else chunk_walk_kernel<16><<<grid, 256, 0, stream>>>(p);
  HFEE_CHECK_LAUNCH("linear_chunks (walk)");
  return 0;
}
