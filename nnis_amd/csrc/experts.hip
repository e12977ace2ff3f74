// The products of a routed feed-forward whose experts are gated: which experts' weights are read follows the router's
// choice.  bfloat16 on the matrix cores with 32-bit sums, weights packed (common.h).
//
// Weights.  Regions 0 .. experts - 1 are the experts, region `experts` is a shared expert that every token uses with
// weight one (absent where its size is 0).  An inner size is padded to a multiple of 64 channels with zeros (kept so
// by both projections), so that regions begin at strips of `up` and at chunks of `down`:
//   up    [experts x (gate rows | up rows) | shared gate rows | shared up rows][width]
//   down  [width][experts x inner | shared inner]
// The shared expert's weight may be a number a token instead of one (`shared_weights` [tokens]).
// Between the two, a region's value is weight * act(gate, up), act by `form`: 1 silu(a) u; 2 the clamped gate
// a sigmoid(1.702 a) (u + 1) with a held at most at the region's limit and u within plus or minus it (0: not held).
//
// Two ways through:
//  * few tokens (up to 16, one tile): `up` and `down` are products with every token, of which the regions that no token
//    chose are left out: nothing of them is read.  hidden [tokens][all inner]: zero where a token did not choose.
//  * many tokens: an expert's products run over the tokens that chose it, gathered by a list.  A pair p = token * top +
//    choice has a row of its own in hidden and in the output; the rows of a token are added to the stream at the end.
#include "common.h"
#include "product.h"

#include <type_traits>

thread_local char g_nnis_error[512] = {0};
extern "C" const char* nnis_last_error() { return g_nnis_error; }

namespace {

typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;

struct Regions {
  int experts, inner;         // inner size of an expert, padded
  int shared;                 // of the shared expert, padded; 0: none
  int form;
  float limit, shared_limit;  // 0: not held
};

__device__ __forceinline__ float gated_value(const Regions& g, float a, float u, float limit) {
  if (g.form == 2) {
    if (limit > 0.0f) {
      a = fminf(a, limit);
      u = fminf(fmaxf(u, -limit), limit);
    }
    return a * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(a * (-1.702f * 1.4426950408889634f))) * (u + 1.0f);
  }
  return a * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(a * -1.4426950408889634f)) * u;
}

// -----------------------------------------------------------------------------
// Few tokens: m <= 16.
// -----------------------------------------------------------------------------
constexpr int kMostExperts = 1024;

// A block of KSPLIT waves takes 16 channels of a region: their gate and their up strip, K dealt to the waves chunk by
// chunk.  gates [m][experts]: zero where a token did not choose; a region that nobody chose is left as it is (the down
// product does not read it).
template <int KSPLIT>
__global__ __launch_bounds__(64 * KSPLIT) void experts_up_few_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ w,
                                                                     const float* __restrict__ gates, const float* __restrict__ shared_weights,
                                                                     bf16_t* __restrict__ hidden, Regions reg, int m, int k) {
  __shared__ float partial[KSPLIT][2][kWave][4];
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, r = lane % 16, g = lane / 16;
  const int units = reg.inner / 16, shared_units = reg.shared / 16;
  const bool is_shared = (int)blockIdx.x < shared_units;  // (the shared expert's blocks first: they wait for nobody's choice)
  const int item = (int)blockIdx.x - shared_units;
  const int region = is_shared ? reg.experts : item / units;
  const int unit = is_shared ? (int)blockIdx.x : item % units;
  float weight = 1.0f;
  if (!is_shared) {
    weight = r < m ? gates[(size_t)r * reg.experts + region] : 0.0f;
    if (!__any(weight != 0.0f)) return;  // (all waves of the block see the same)
  } else if (shared_weights) {
    weight = r < m ? shared_weights[r] : 0.0f;
  }
  const int strip = is_shared ? reg.experts * 2 * units + unit : region * 2 * units + unit;
  const int strip_up = strip + (is_shared ? shared_units : units);
  const int chunks = nnis_packed_chunks(k);
  const bf16_t* w_gate = w + nnis_packed_lane(strip * 16 + r, g, k);
  const bf16_t* w_up = w + nnis_packed_lane(strip_up * 16 + r, g, k);
  const bf16_t* x_row = x + (size_t)(r < m ? r : m - 1) * k;
  f32x4 acc[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}};
  constexpr int DEPTH = 4;
  for (int base = wave; base < chunks; base += KSPLIT * DEPTH) {
    bf16x8 wg[DEPTH][2], wu[DEPTH][2], xv[DEPTH][2];
#pragma unroll
    for (int d = 0; d < DEPTH; ++d) {
      const int c = base + d * KSPLIT;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const size_t at = (size_t)c * kPackedChunkElems + half * kPackedHalfElems;
        wg[d][half] = c < chunks ? load_chunk(w_gate + at) : zero_chunk();
        wu[d][half] = c < chunks ? load_chunk(w_up + at) : zero_chunk();
      }
    }
#pragma unroll
    for (int d = 0; d < DEPTH; ++d) {
      const int kk = (base + d * KSPLIT) * 64 + g * 16;
      xv[d][0] = kk + 8 <= k ? load_chunk(x_row + kk) : zero_chunk();
      xv[d][1] = kk + 16 <= k ? load_chunk(x_row + kk + 8) : zero_chunk();
    }
#pragma unroll
    for (int d = 0; d < DEPTH; ++d)
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        acc[0] = mfma(wg[d][half], xv[d][half], acc[0]);
        acc[1] = mfma(wu[d][half], xv[d][half], acc[1]);
      }
  }
  if (wave != 0) {
#pragma unroll
    for (int p = 0; p < 2; ++p) *(f32x4*)&partial[wave][p][lane][0] = acc[p];
  }
  __syncthreads();
  if (wave != 0) return;
#pragma unroll
  for (int other = 1; other < KSPLIT; ++other)
#pragma unroll
    for (int p = 0; p < 2; ++p) acc[p] += *(const f32x4*)&partial[other][p][lane][0];
  if (r >= m) return;
  const float limit = is_shared ? reg.shared_limit : reg.limit;
  bf16x4 out;
#pragma unroll
  for (int e = 0; e < 4; ++e) out[e] = (__bf16)(weight == 0.0f ? 0.0f : weight * gated_value(reg, acc[0][e], acc[1][e], limit));
  const size_t row = (size_t)r * (reg.experts * reg.inner + reg.shared);
  *(bf16x4*)(hidden + row + (size_t)region * reg.inner + unit * 16 + 4 * g) = out;
}

// Two blocks of KSPLIT waves take 16 output channels between them (the strips alone would leave half the chip without a block)
// and meet as the library's paired products do: the chunks of the regions that somebody chose, and of the shared one,
// dealt to the waves of both.
template <int KSPLIT, typename OutT>
__global__ __launch_bounds__(64 * KSPLIT) void experts_down_few_kernel(const bf16_t* __restrict__ hidden, const bf16_t* __restrict__ w,
                                                                       const float* __restrict__ gates, OutT y, Regions reg, int m, int n,
                                                                       PairScratch pair) {
  constexpr int kShares = 2 * KSPLIT;
  __shared__ float partial[KSPLIT][kWave][4];
  __shared__ short active[kMostExperts];
  __shared__ int active_count;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, r = lane % 16, g = lane / 16;
  const int strip = blockIdx.x / 2, share = 2 * wave + (int)(blockIdx.x % 2);
  const int k = reg.experts * reg.inner + reg.shared;
  constexpr bool kResidual = std::is_same<OutT, ResidualOut>::value;
  const int n0 = strip * 16 + g * 4;
  const int valid = r < m ? (n - n0 >= 4 ? 4 : (n - n0 > 0 ? n - n0 : 0)) : 0;
  const bool vector_ok = (n % 4) == 0;
  ResidualHeld held;
  if constexpr (kResidual) {
    if (wave == 0) held = residual_ask(y, (size_t)(r < m ? r : 0) * n + (valid > 0 ? n0 : 0), valid > 0 ? n0 : 0, valid, vector_ok);
  }
  if (wave == KSPLIT - 1) {  // the regions somebody chose, in order
    int count = 0;
    for (int e0 = 0; e0 < reg.experts; e0 += kWave) {
      const int e = e0 + lane;
      float any = 0.0f;
#pragma unroll
      for (int t = 0; t < 16; ++t) any = fmaxf(any, fabsf(gates[(size_t)(t < m ? t : m - 1) * reg.experts + (e < reg.experts ? e : 0)]));
      const unsigned long long mask = __ballot(e < reg.experts && any != 0.0f);
      if (mask >> lane & 1ull) active[count + __popcll(mask & ((1ull << lane) - 1ull))] = (short)e;
      count += __popcll(mask);
    }
    if (lane == 0) active_count = count;
  }
  const bf16_t* w_ptr = w + nnis_packed_lane(strip * 16 + r, g, k);
  const bf16_t* x_row = hidden + (size_t)(r < m ? r : m - 1) * k + g * 16;
  __syncthreads();
  const int per = reg.inner / 64, shared_chunks = reg.shared / 64;
  const int chunks = active_count * per + shared_chunks;
  f32x4 sums[1] = {{0.0f, 0.0f, 0.0f, 0.0f}};
  f32x4& acc = sums[0];
  constexpr int DEPTH = 4;
  for (int base = share; base < chunks; base += kShares * DEPTH) {
    bf16x8 wv[DEPTH][2], xv[DEPTH][2];
#pragma unroll
    for (int d = 0; d < DEPTH; ++d) {
      int c = base + d * kShares;
      const bool inside = c < chunks;
      c = inside ? c : chunks - 1;
      // the shared expert's chunks first, then the chosen regions'
      c = c < shared_chunks ? reg.experts * per + c : active[(c - shared_chunks) / per] * per + (c - shared_chunks) % per;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        wv[d][half] = inside ? load_chunk(w_ptr + (size_t)c * kPackedChunkElems + half * kPackedHalfElems) : zero_chunk();
        xv[d][half] = inside ? load_chunk(x_row + (size_t)c * 64 + 8 * half) : zero_chunk();
      }
    }
#pragma unroll
    for (int d = 0; d < DEPTH; ++d)
#pragma unroll
      for (int half = 0; half < 2; ++half) acc = mfma(wv[d][half], xv[d][half], acc);
  }
  if (wave != 0) *(f32x4*)&partial[wave][lane][0] = acc;
  __syncthreads();
  if (wave != 0) return;
#pragma unroll
  for (int other = 1; other < KSPLIT; ++other) acc += *(const f32x4*)&partial[other][lane][0];
  if (!pair_meets<1>(sums, pair, strip, blockIdx.x % 2, lane)) return;  // the first of the two: the other ends the strip
  if constexpr (kResidual) {
    float sq = 0.0f;
    if (valid > 0) sq = residual_take(y, held, (size_t)r * n + n0, acc, valid, vector_ok);
    sq += __shfl_xor(sq, 16, kWave);
    sq += __shfl_xor(sq, 32, kWave);
    if (g == 0 && r < m) y.ss[(size_t)strip * m + r] = sq;
  } else {
    if (valid > 0) store4(y, (size_t)r * n + n0, acc, valid, vector_ok);
  }
}

// -----------------------------------------------------------------------------
// Many tokens.
// -----------------------------------------------------------------------------

// lists [experts][tokens]: the pairs (token * top + choice) of the tokens that chose an expert, in the tokens' order;
// counts [experts].  A block an expert.
__global__ __launch_bounds__(1024) void experts_lists_kernel(const int* __restrict__ chosen, int tokens, int top, int* __restrict__ counts,
                                                            int* __restrict__ lists) {
  __shared__ int waves_before[17];
  const int e = blockIdx.x, wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, waves = blockDim.x / kWave;
  int* list = lists + (size_t)e * tokens;
  int total = 0;
  for (int t0 = 0; t0 < tokens; t0 += blockDim.x) {
    const int t = t0 + threadIdx.x;
    int pair = -1;
    if (t < tokens)
      for (int c = 0; c < top; ++c)
        if (chosen[(size_t)t * top + c] == e) pair = t * top + c;
    const unsigned long long mask = __ballot(pair >= 0);
    __syncthreads();  // (the round before has read its counts)
    if (lane == 0) waves_before[wave] = __popcll(mask);
    __syncthreads();
    int before = total;
    for (int o = 0; o < waves; ++o) {
      const int here = waves_before[o];
      if (o < wave) before += here;
      total += here;
    }
    if (pair >= 0) list[before + __popcll(mask & ((1ull << lane) - 1ull))] = pair;
  }
  if (threadIdx.x == 0) counts[e] = total;
}

typedef __attribute__((address_space(1))) const void* global_ptr_t;
typedef __attribute__((address_space(3))) void* lds_ptr_t;
// The loads into LDS are not the compiler's to wait for: the kernel counts them itself.
template <int N>
__device__ __forceinline__ void wait_loads_but() { asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory"); }

extern __shared__ __align__(16) char tile_lds[];

struct ManyArgs {
  const bf16_t* x;         // UP: the tokens' rows [tokens][width]; DOWN: the pairs' hidden rows [tokens * top][inner]
  const bf16_t* x_shared;  // DOWN: the shared expert's hidden rows [tokens][shared]
  const bf16_t* w;
  bf16_t* y;               // UP: hidden rows of the pairs; DOWN: the pairs' outputs [tokens * top][width]
  bf16_t* y_shared;        // of the shared expert: [tokens][shared] or [tokens][width]
  const float* weights;    // [tokens * top]
  const float* shared_weights;  // [tokens] or null: ones
  const int* counts;
  const int* lists;
  Regions reg;
  int tokens, top, width;
  int run;                 // column blocks that a block takes one after the other
};

// A block of 8 waves takes 128 of a region's rows and BN weight rows -- UP: BN / 2 channels' gate and up rows, strips
// alternating between the two -- through a ring of three stages of 64 k in LDS, as the library's tiled product does
// (operands straight from memory into LDS, activations' chunks of 16 bytes swizzled by row; a step's second half is
// multiplied behind the barrier).  The rows are gathered: a row's address is its list entry's.
// The wide tile brings three quarters of the narrow one's bytes through L2 a multiplication; the narrow one fills the chip
// with few rows.  Up and down product of 16 experts of 704, 2 chosen, and a shared one of 1,408 on rows of 2,048 channels,
// microseconds, narrow and wide: 192 rows 25 + 25 / 34 + 26; with two stages of the narrow one, two blocks a unit, against the
// wide one: 512 rows 40 + 30 / 35 + 27, 2,048 rows 80 + 56 / 72 + 50, 8,192 rows 243 + 193 / 208 + 166.
// An item is a row block and a run of `run` column blocks: the ring goes on from one to the next, so that the next one's loads
// are under way while the last one's rows go out, and a short K (an expert's inner size) pays for its beginning once.  Items
// are dealt so that a die runs a run of neighbours, the row blocks of one block of weights one after another.
template <bool UP, int BN>
__global__ __launch_bounds__(512) void experts_tiled_kernel(ManyArgs a) {
  constexpr int BM = 128, BK = 64, NS = 3, W = 8, WGN = BN / 64;
  constexpr int WM = BM * WGN / W, WN = 64, TM = WM / 16, TN = WN / 16;
  constexpr int CHANNELS = BN / 2;  // UP: of a tile
  constexpr int A_LOADS = BM / (8 * W), B_LOADS = BN / (8 * W), LOADS = A_LOADS + B_LOADS;
  constexpr int A_BYTES = BM * BK * 2, STAGE_BYTES = (BM + BN) * BK * 2;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid / kWave), lane = tid % kWave;
  const int wave_m = wave / WGN, wave_n = wave % WGN, r = lane % 16, g = lane / 16;
  const Regions& reg = a.reg;
  // which item: the regions' row blocks are counted from the lists' lengths (every wave for itself)
  const int cols = UP ? (reg.inner + CHANNELS - 1) / CHANNELS : (a.width + BN - 1) / BN;
  const int cols_shared = reg.shared == 0 ? 0 : (UP ? (reg.shared + CHANNELS - 1) / CHANNELS : cols);
  const int runs = (cols + a.run - 1) / a.run;
  const int shared_items = (a.tokens + BM - 1) / BM * ((cols_shared + a.run - 1) / a.run);
  int total = shared_items;
  for (int e0 = 0; e0 < reg.experts; e0 += kWave) {
    const int e = e0 + lane;
    int blocks = e < reg.experts ? (a.counts[e] + BM - 1) / BM : 0;
#pragma unroll
    for (int offset = kWave / 2; offset > 0; offset >>= 1) blocks += __shfl_xor(blocks, offset, kWave);
    total += blocks * runs;
  }
  total = __builtin_amdgcn_readfirstlane(total);
  int item;
  {
    const int die = blockIdx.x % 8, nth = blockIdx.x / 8;
    const int each = total / 8, more = total % 8;
    if (nth >= each + (die < more ? 1 : 0)) return;  // (the grid is as large as any choice of the router can make it)
    item = die * each + (die < more ? die : more) + nth;
  }
  int region = reg.experts, rows = a.tokens, blocks_here = (a.tokens + BM - 1) / BM;
  if (item >= shared_items) {
    item -= shared_items;
    int before = 0;
    for (int e0 = 0; e0 < reg.experts; e0 += kWave) {
      const int e = e0 + lane;
      const int count = e < reg.experts ? a.counts[e] : 0;
      const int items = (count + BM - 1) / BM * runs;
      int upto = items;  // inclusive sum over the lanes
#pragma unroll
      for (int offset = 1; offset < kWave; offset <<= 1) {
        const int other = __shfl_up(upto, offset, kWave);
        if (lane >= offset) upto += other;
      }
      upto += before;
      const unsigned long long found = __ballot(item < upto);
      if (found) {
        const int at = __ffsll(found) - 1;
        region = e0 + at;
        rows = __shfl(count, at, kWave);
        item -= __shfl(upto - items, at, kWave);
        break;
      }
      before = __shfl(upto, kWave - 1, kWave);
    }
    blocks_here = (rows + BM - 1) / BM;
  }
  region = __builtin_amdgcn_readfirstlane(region);
  rows = __builtin_amdgcn_readfirstlane(rows);
  item = __builtin_amdgcn_readfirstlane(item);
  blocks_here = __builtin_amdgcn_readfirstlane(blocks_here);
  const bool is_shared = region == reg.experts;
  const int row0 = (item % blocks_here) * BM, col0 = item / blocks_here * a.run;
  const int col_end = min(col0 + a.run, is_shared ? cols_shared : cols);
  const int* list = is_shared ? nullptr : a.lists + (size_t)region * a.tokens;
  const int k = UP ? a.width : (is_shared ? reg.shared : reg.inner);           // of this product
  const int w_k = UP ? a.width : reg.experts * reg.inner + reg.shared;         // of the packed weight's rows
  const int first_chunk = UP ? 0 : region * (reg.inner / 64);                  // (the shared region lies behind the experts')

  const bf16_t* a_src[A_LOADS];
  const bf16_t* b_src[B_LOADS];
  const int chunk_k = ((lane % 8) ^ (lane / 8)) * 8;
#pragma unroll
  for (int o = 0; o < A_LOADS; ++o) {
    int row = row0 + (o * W + wave) * 8 + lane / 8;
    row = row < rows ? row : rows - 1;
    const int from = list ? list[row] : row;
    const bf16_t* base = UP ? a.x + (size_t)(list ? from / a.top : from) * k : (is_shared ? a.x_shared : a.x) + (size_t)from * k;
    a_src[o] = base + chunk_k;
  }
  const int channels = is_shared ? reg.shared : reg.inner;  // UP: channels of the region
  const int gate_row = UP ? (is_shared ? reg.experts * 2 * reg.inner : region * 2 * reg.inner) : 0;
  auto take_column = [&](int col) {  // the weight rows of a column block
#pragma unroll
    for (int o = 0; o < B_LOADS; ++o) {
      const int piece = o * W + wave, strip = piece / 2;
      int row;
      if (UP) {
        int unit = col * CHANNELS + (strip / 2) * 16;  // (a tile's channels beyond the region's: multiplied again from its last, not stored)
        unit = unit < channels ? unit : channels - 16;
        row = gate_row + (strip % 2 ? channels : 0) + unit + r;
      } else {
        row = col * BN + strip * 16 + r;
        row = row < a.width ? row : a.width - 1;
      }
      b_src[o] = a.w + nnis_packed_lane(row, g, w_k) + (size_t)first_chunk * kPackedChunkElems + (piece % 2) * kPackedHalfElems;
    }
  };
  take_column(col0);
  const int steps = (k + BK - 1) / BK;
  int last_chunk = k - 8 - chunk_k;  // offset of the row's last whole chunk from this lane's first
  last_chunk = last_chunk > -chunk_k ? last_chunk : -chunk_k;
  int ask_step = 0, ask_col = col0;  // what is asked for next
  auto ask = [&](int stage) {
    char* base = tile_lds + stage * STAGE_BYTES + wave * 1024;
    const int k0 = ask_step * BK;
    const int from = k0 <= last_chunk ? k0 : last_chunk;
#pragma unroll
    for (int o = 0; o < A_LOADS; ++o)
      __builtin_amdgcn_global_load_lds((global_ptr_t)(a_src[o] + from), (lds_ptr_t)(base + o * W * 1024), 16, 0, 0);
    const size_t from_chunk = (size_t)ask_step * kPackedChunkElems;
#pragma unroll
    for (int o = 0; o < B_LOADS; ++o)
      __builtin_amdgcn_global_load_lds((global_ptr_t)(b_src[o] + from_chunk), (lds_ptr_t)(base + A_BYTES + o * W * 1024), 16, 0, 0);
    if (ask_step + 1 < steps) ++ask_step;
    else if (ask_col + 1 < col_end) take_column(++ask_col), ask_step = 0;
    // (beyond the last column block: its last step again, a valid address that nobody reads, so that the count of loads holds)
  };
  f32x4 acc[TM][TN];
#pragma unroll
  for (int i = 0; i < TM; ++i)
#pragma unroll
    for (int j = 0; j < TN; ++j) acc[i][j] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
  for (int s = 0; s < NS - 1; ++s) ask(s);
  // the rows this lane ends up with, asked for behind the first steps' loads
  int out_row[TM];
  float weight[TM];
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    int row = row0 + wave_m * WM + i * 16 + r;
    const bool live = row < rows;
    row = live ? row : rows - 1;
    const int to = list ? list[row] : row;
    weight[i] = UP ? 1.0f : (list ? a.weights[to] : (a.shared_weights ? a.shared_weights[to] : 1.0f));
    out_row[i] = live ? to : -1;
  }
  wait_loads_but<0>();
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
  bf16x8 a0[TM], b0[TN], a1[TM], b1[TN];
  auto read_half = [&](int from, int half, bf16x8 (&av)[TM], bf16x8 (&bv)[TN]) {
    const bf16x8* a_tile = (const bf16x8*)(tile_lds + from * STAGE_BYTES);
    const bf16x8* b_tile = (const bf16x8*)(tile_lds + from * STAGE_BYTES + A_BYTES);
#pragma unroll
    for (int i = 0; i < TM; ++i) {
      const int row = wave_m * WM + i * 16 + r;
      av[i] = a_tile[row * 8 + ((g * 2 + half) ^ (row & 7))];
    }
#pragma unroll
    for (int j = 0; j < TN; ++j) bv[j] = b_tile[((wave_n * TN + j) * 2 + half) * kWave + lane];
  };
  auto multiply = [&](const bf16x8 (&av)[TM], const bf16x8 (&bv)[TN]) {
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
      for (int j = 0; j < TN; ++j) acc[i][j] = mfma(bv[j], av[i], acc[i][j]);
  };
  auto interleave = [&]() {  // for the scheduler: a read behind each of the first products, then the rest of the products
#pragma unroll
    for (int n = 0; n < TM + TN; ++n) {
      __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x008, TM * TN - (TM + TN), 0);
  };
  const float limit = is_shared ? reg.shared_limit : reg.limit;
  bf16_t* y = is_shared ? a.y_shared : a.y;
  const bool vector_ok = a.width % 4 == 0;
  auto put = [&](int col) {  // a finished tile's rows; the sums begin again
#pragma unroll
    for (int i = 0; i < TM; ++i) {
      if (out_row[i] < 0) continue;
      if (UP) {
#pragma unroll
        for (int u = 0; u < TN / 2; ++u) {
          const int unit = col * CHANNELS + wave_n * 32 + u * 16;
          if (unit >= channels) continue;
          bf16x4 out;
#pragma unroll
          for (int e = 0; e < 4; ++e) out[e] = (__bf16)gated_value(reg, acc[i][2 * u][e], acc[i][2 * u + 1][e], limit);
          *(bf16x4*)(y + (size_t)out_row[i] * channels + unit + 4 * g) = out;
        }
      } else {
#pragma unroll
        for (int j = 0; j < TN; ++j) {
          const int n0 = col * BN + wave_n * WN + j * 16 + 4 * g;
          const int valid = a.width - n0 >= 4 ? 4 : (a.width - n0 > 0 ? a.width - n0 : 0);
          if (valid > 0) store4(y, (size_t)out_row[i] * a.width + n0, acc[i][j] * weight[i], valid, vector_ok);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
      for (int j = 0; j < TN; ++j) acc[i][j] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
  };
  // (A column block's stores stand between two steps' loads in the order in which the counter below sees them end: the
  // step after waits for them too, by when they have had a step's time.)
  int stage = 0;
  read_half(0, 0, a0, b0);
  for (int col = col0; col < col_end; ++col) {
    for (int step = 0; step < steps; ++step) {
      ask(stage == 0 ? NS - 1 : stage - 1);
      read_half(stage, 1, a1, b1);
      multiply(a0, b0);
      interleave();
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      wait_loads_but<(NS - 2) * LOADS>();
      __builtin_amdgcn_sched_barrier(0);
      __builtin_amdgcn_s_barrier();
      __builtin_amdgcn_sched_barrier(0);
      asm volatile("" ::: "memory");
      stage = stage + 1 == NS ? 0 : stage + 1;
      read_half(stage, 0, a0, b0);  // (after the last step: of a stage that nobody multiplies)
      multiply(a1, b1);
      interleave();
    }
    put(col);
  }
  wait_loads_but<0>();  // the steps asked for beyond the end: nothing of this block is in flight when it ends
}

// The end: a token's pairs and its shared row added up, into the stream with the norm that follows prepared (ResidualOut:
// one part of a row's sum of squares), or stored.  A block a token.
template <typename OutT>
__global__ __launch_bounds__(256) void experts_combine_kernel(const bf16_t* __restrict__ pairs, const bf16_t* __restrict__ shared, OutT y, int tokens,
                                                             int top, int width) {
  __shared__ float scratch[16];
  constexpr bool kResidual = std::is_same<OutT, ResidualOut>::value;
  const int token = blockIdx.x;
  float sq = 0.0f;
  const bool vector_ok = width % 4 == 0;
  for (int c = 4 * threadIdx.x; c < width; c += 4 * blockDim.x) {
    const int valid = width - c >= 4 ? 4 : width - c;
    const size_t index = (size_t)token * width + c;
    ResidualHeld held;
    if constexpr (kResidual) held = residual_ask(y, index, c, valid, vector_ok);
    f32x4 sum = {0.0f, 0.0f, 0.0f, 0.0f};
    auto take = [&](const bf16_t* row) {
      if (valid == 4 && vector_ok) {
        const bf16x4 v = *(const bf16x4*)(row + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) sum[e] += (float)v[e];
      } else {
        for (int e = 0; e < valid; ++e) sum[e] += (float)row[c + e];
      }
    };
#pragma unroll 2
    for (int p = 0; p < top; ++p) take(pairs + ((size_t)token * top + p) * width);
    if (shared) take(shared + (size_t)token * width);
    if constexpr (kResidual) sq += residual_take(y, held, index, sum, valid, vector_ok);
    else store4(y, index, sum, valid, vector_ok);
  }
  if constexpr (kResidual) {
    sq = block_sum(sq, scratch);
    if (threadIdx.x == 0) y.ss[token] = sq;
  }
}

int check_regions(const char* what, const Regions& reg) {
  NNIS_REQUIRE(reg.experts > 0 && reg.experts <= kMostExperts && reg.inner > 0 && reg.inner % 64 == 0 && reg.shared >= 0 && reg.shared % 64 == 0,
               "%s: 1 to %d experts of a size in steps of 64 (and a shared one); got %d of %d, shared %d", what, kMostExperts, reg.experts, reg.inner,
               reg.shared);
  NNIS_REQUIRE(reg.form == 1 || reg.form == 2, "%s: unknown form %d", what, reg.form);
  return 0;
}

}  // namespace

// x [m, k] bfloat16, gates float32 [m, experts], shared_weights float32 [m] or null, hidden [m, experts * inner + shared]; m <= 16
extern "C" int nnis_experts_up_few(const void* x, const void* w, const float* gates, const float* shared_weights, void* hidden, int m, int k, int experts, int inner, int shared,
                                   int form, float limit, float shared_limit, void* stream) {
  const Regions reg = {experts, inner, shared, form, limit, shared_limit};
  if (check_regions("experts_up_few", reg)) return 1;
  NNIS_REQUIRE(x && w && gates && hidden && m >= 0 && m <= 16 && k > 0 && k % 8 == 0, "experts_up_few: up to 16 rows of a multiple of 8 channels, got %d of %d",
               m, k);
  NNIS_REQUIRE((uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)hidden % 16 == 0, "experts_up_few: operands must be 16-byte aligned");
  if (m == 0) return 0;
  const unsigned blocks = (unsigned)(experts * (inner / 16) + shared / 16);
  const int chunks = nnis_packed_chunks(k);
  hipStream_t s = (hipStream_t)stream;
#define NNIS_UP_FEW(SPLIT_)                                                                                                          \
  hipLaunchKernelGGL((experts_up_few_kernel<SPLIT_>), dim3(blocks), dim3(64 * SPLIT_), 0, s, (const bf16_t*)x, (const bf16_t*)w, gates, \
                     shared_weights, (bf16_t*)hidden, reg, m, k)
  // (rows of 2,048 channels, 16 experts of 704: 11 of them chosen 17.7 us with 8 waves, 19.8 with 4 and 20.7 with 16; 2 of them
  // 7.8, 6.3 and 8.1)
  if (chunks > 16 && m > 2) NNIS_UP_FEW(8);
  else if (chunks > 4) NNIS_UP_FEW(4);
  else NNIS_UP_FEW(2);
#undef NNIS_UP_FEW
  NNIS_LAUNCH_CHECK("experts_up_few");
  return 0;
}

// hidden as above, the product [m, n] into y: bfloat16 rows (resid null), or into the stream with the following norm prepared
// (resid float32 [m, n], gain, scaled bfloat16 [m, n], ss float32 [(n + 15) / 16, m]).  pair_sums: scratch of 2 KB a strip of 16
// channels; pair_counts: a word a strip, zero between calls; pair_strips: for how many strips both are.
extern "C" int nnis_experts_down_few(const void* hidden, const void* w, const float* gates, void* y, float* resid, const void* gain, int gain_dtype,
                                     void* scaled, float* ss, int m, int n, int experts, int inner, int shared, int form, float* pair_sums,
                                     int* pair_counts, int pair_strips, void* stream) {
  const Regions reg = {experts, inner, shared, form, 0.0f, 0.0f};
  if (check_regions("experts_down_few", reg)) return 1;
  NNIS_REQUIRE(hidden && w && gates && m >= 0 && m <= 16 && n > 0, "experts_down_few: up to 16 rows, got %d", m);
  NNIS_REQUIRE(resid ? (gain && scaled && ss && nnis_dtype_ok(gain_dtype)) : y != nullptr, "experts_down_few: nowhere to put the product");
  NNIS_REQUIRE((uintptr_t)hidden % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)resid % 16 == 0 &&
                   (uintptr_t)scaled % 16 == 0 && (uintptr_t)gain % 16 == 0,
               "experts_down_few: operands must be 16-byte aligned");
  const unsigned strips = (unsigned)((n + 15) / 16);
  NNIS_REQUIRE(pair_sums && pair_counts && (int)strips <= pair_strips, "experts_down_few: scratch for %u strips is needed, not %d", strips, pair_strips);
  if (m == 0) return 0;
  const PairScratch pair = {pair_sums, pair_counts};
  hipStream_t s = (hipStream_t)stream;
  if (resid) {
    ResidualOut out;
    out.resid = resid; out.gain = gain; out.gain_dtype = gain_dtype; out.scaled = (bf16_t*)scaled; out.ss = ss;
    hipLaunchKernelGGL((experts_down_few_kernel<8, ResidualOut>), dim3(2 * strips), dim3(64 * 8), 0, s, (const bf16_t*)hidden, (const bf16_t*)w, gates,
                       out, reg, m, n, pair);
  } else {
    hipLaunchKernelGGL((experts_down_few_kernel<8, bf16_t*>), dim3(2 * strips), dim3(64 * 8), 0, s, (const bf16_t*)hidden, (const bf16_t*)w, gates,
                       (bf16_t*)y, reg, m, n, pair);
  }
  NNIS_LAUNCH_CHECK("experts_down_few");
  return 0;
}

// chosen int32 [tokens, top] -> counts int32 [experts], lists int32 [experts, tokens]
extern "C" int nnis_experts_lists(const int* chosen, int tokens, int top, int experts, int* counts, int* lists, void* stream) {
  NNIS_REQUIRE(chosen && counts && lists && top > 0 && experts > 0 && tokens >= 0, "experts_lists: missing operand");
  NNIS_REQUIRE((long long)tokens * top <= 0x7fffffff, "experts_lists: too many pairs");
  hipLaunchKernelGGL(experts_lists_kernel, dim3(experts), dim3(1024), 0, (hipStream_t)stream, chosen, tokens, top, counts, lists);
  NNIS_LAUNCH_CHECK("experts_lists");
  return 0;
}

// which 0: `up`, x [tokens, width] -> y [tokens * top, inner], y_shared [tokens, shared];
// which 1: `down`, x [tokens * top, inner], x_shared [tokens, shared] -> y [tokens * top, width] (each row times its pair's
// weight, the shared expert's times its token's shared_weights where given), y_shared [tokens, width].  Rows whose pair chose no expert of the lists do not exist: every pair has its expert.
extern "C" int nnis_experts_many(int which, const void* x, const void* x_shared, const void* w, void* y, void* y_shared, const float* weights,
                                 const float* shared_weights, const int* counts, const int* lists, int tokens, int top, int width, int experts, int inner, int shared, int form,
                                 float limit, float shared_limit, void* stream) {
  const Regions reg = {experts, inner, shared, form, limit, shared_limit};
  if (check_regions("experts_many", reg)) return 1;
  NNIS_REQUIRE(x && w && y && weights && counts && lists && tokens >= 0 && top > 0 && top <= experts && width > 0 && width % 8 == 0,
               "experts_many: missing operand or bad sizes (top %d, width %d)", top, width);
  NNIS_REQUIRE(shared == 0 || (y_shared && (which == 0 || x_shared)), "experts_many: the shared expert's rows are missing");
  for (const void* p : {x, x_shared, w, (const void*)y, (const void*)y_shared})
    NNIS_REQUIRE((uintptr_t)p % 16 == 0, "experts_many: operands must be 16-byte aligned");
  if (tokens == 0) return 0;
  // row blocks of 128: as many as any choice can make
  const long long pairs = (long long)tokens * top;
  long long row_blocks = pairs / 128 + (experts < pairs ? experts : pairs);
  const bool wide = tokens > 320;
  const long long tile = wide ? 256 : 128;
  const long long cols = which == 0 ? (inner + tile / 2 - 1) / (tile / 2) : (width + tile - 1) / tile;
  const long long cols_shared = shared == 0 ? 0 : (which == 0 ? (shared + tile / 2 - 1) / (tile / 2) : cols);
  const long long shared_rows = (tokens + 127) / 128;
  // How many column blocks a block takes, one or two: what leaves the fewest (rounds of blocks) x (an item's steps and its beginning
  // and end, worth eight steps), for the row blocks that a fairly even choice makes.  (The sizes above at 2,048 rows, one and two: 76
  // + 50 us and 67 + 48; in longer runs, at 4,096 and 8,192 rows, what one product gained the other lost.)
  const long long likely_rows = pairs / 128 + (experts < pairs ? experts : pairs) / 2;
  const long long steps = which == 0 ? (width + 63) / 64 : inner / 64;
  long long run = 1, best = -1;
  for (long long r = 1; r <= 2; ++r) {
    const long long items = likely_rows * ((cols + r - 1) / r) + shared_rows * ((cols_shared + r - 1) / r);
    const long long cost = (items + 255) / 256 * (r * steps + 8);
    if (best < 0 || cost < best) best = cost, run = r;
  }
  long long blocks = row_blocks * ((cols + run - 1) / run) + shared_rows * ((cols_shared + run - 1) / run);
  blocks = (blocks + 7) / 8 * 8;
  NNIS_REQUIRE(blocks <= 0x7fffffff, "experts_many: the step exceeds the grid limit");
  ManyArgs a;
  a.x = (const bf16_t*)x; a.x_shared = (const bf16_t*)x_shared; a.w = (const bf16_t*)w; a.y = (bf16_t*)y; a.y_shared = (bf16_t*)y_shared;
  a.weights = weights; a.shared_weights = shared_weights; a.counts = counts; a.lists = lists; a.reg = reg; a.tokens = tokens; a.top = top; a.width = width;
  a.run = (int)run;
  hipStream_t s = (hipStream_t)stream;
  // (beyond 64 KB a kernel has to be told once; a refusal shows as the launch's failure)
#define NNIS_EXPERTS_TILED(UP_, BN_)                                                                                          \
  do {                                                                                                                        \
    constexpr int lds_bytes = 3 * (128 + BN_) * 64 * 2;                                                                       \
    static const hipError_t allowed = hipFuncSetAttribute((const void*)experts_tiled_kernel<UP_, BN_>,                        \
                                                          hipFuncAttributeMaxDynamicSharedMemorySize, lds_bytes);             \
    (void)allowed;                                                                                                            \
    hipLaunchKernelGGL((experts_tiled_kernel<UP_, BN_>), dim3((unsigned)blocks), dim3(512), lds_bytes, s, a);                 \
  } while (0)
  if (which == 0 && wide) NNIS_EXPERTS_TILED(true, 256);
  else if (which == 0) NNIS_EXPERTS_TILED(true, 128);
  else if (wide) NNIS_EXPERTS_TILED(false, 256);
  else NNIS_EXPERTS_TILED(false, 128);
#undef NNIS_EXPERTS_TILED
  NNIS_LAUNCH_CHECK("experts_many");
  return 0;
}

// pairs [tokens * top, width] and shared [tokens, width] (null: none), added up per token, into y or the stream (see nnis_experts_down_few;
// ss float32 [1, tokens])
extern "C" int nnis_experts_combine(const void* pairs, const void* shared, void* y, float* resid, const void* gain, int gain_dtype, void* scaled,
                                    float* ss, int tokens, int top, int width, void* stream) {
  NNIS_REQUIRE(pairs && tokens >= 0 && top > 0 && width > 0, "experts_combine: missing operand");
  NNIS_REQUIRE(resid ? (gain && scaled && ss && nnis_dtype_ok(gain_dtype)) : y != nullptr, "experts_combine: nowhere to put the sum");
  for (const void* p : {pairs, shared, (const void*)y, (const void*)resid, gain, (const void*)scaled})
    NNIS_REQUIRE((uintptr_t)p % 16 == 0, "experts_combine: operands must be 16-byte aligned");
  if (tokens == 0) return 0;
  const int threads = width <= 256 ? 64 : (width <= 512 ? 128 : 256);
  hipStream_t s = (hipStream_t)stream;
  if (resid) {
    ResidualOut out;
    out.resid = resid; out.gain = gain; out.gain_dtype = gain_dtype; out.scaled = (bf16_t*)scaled; out.ss = ss;
    hipLaunchKernelGGL((experts_combine_kernel<ResidualOut>), dim3(tokens), dim3(threads), 0, s, (const bf16_t*)pairs, (const bf16_t*)shared, out, tokens,
                       top, width);
  } else {
    hipLaunchKernelGGL((experts_combine_kernel<bf16_t*>), dim3(tokens), dim3(threads), 0, s, (const bf16_t*)pairs, (const bf16_t*)shared, (bf16_t*)y,
                       tokens, top, width);
  }
  NNIS_LAUNCH_CHECK("experts_combine");
  return 0;
}
