// Mamba-2's mixer between its projections (state-space duality): a matrix state per head that one number a head and token
// lets decay, and the gated norm in parts behind it.
//
// Rows.  A step's rows are packed: sequence b owns rows seq_start[b] .. seq_start[b + 1] - 1, which continue the sequence in
// slot seq_slot[b] (negative: padding).  `xbc` [tokens, stride] holds, behind the convolution, a token's x (heads * P channels),
// B and C (groups * N each); head h uses group h / (heads / groups).  Per head, S [P, N] (32-bit, column by column of the
// design's [N, P]: a value channel's N states are consecutive) and
//     dt = softplus(z_dt + dt_bias),  S <- exp(-rate dt) S + dt x B^T,  y = S C + D x,   rate = exp(A_log) ready-made
// Decays, step sizes, exponentials, state and sums are 32-bit whatever the storage type.
//
// Three kernels: state_space_scan_kernel, token by token, for any types and sizes; state_space_chunks_kernel, prompts of
// bfloat16 rows on the matrix cores, 64 tokens at a time; state_space_step_kernel, single tokens with the convolution in it.
#include "common.h"

thread_local char g_nnis_error[512] = {0};
extern "C" const char* nnis_last_error() { return g_nnis_error; }

namespace {

constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + exp2_fast(-z * kLog2e)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
// the same by the hardware's 2^x and log2: e^z itself where it is small (1 + e^z would round it away: three terms of the logarithm's
// series, a relative error below 2e-6)
__device__ __forceinline__ float softplus_fast(float z) {
  const float t = exp2_fast(z * kLog2e);
  const float small = t * (1.0f - t * (0.5f - t * (1.0f / 3.0f)));
  const float mid = __builtin_amdgcn_logf(1.0f + t) * 0.6931471805599453f;
  return z > 20.0f ? z : (t < 0.02f ? small : mid);
}

struct SpaceArgs {
  const void* xbc;  // [tokens, xbc_stride]
  int xbc_dtype, xbc_stride;
  const void* dt;  // [tokens, dt_stride]: z_dt of every head
  int dt_dtype, dt_stride;
  const float* rate;     // [heads]
  const float* dt_bias;  // [heads]
  const float* D;        // [heads]
  const void* z;  // [tokens, z_stride]: y leaves times silu(z)
  int z_dtype, z_stride;
  float* state;  // [slots, heads, P, N]
  const int* seq_slot;
  const int* seq_start;
  int heads, groups, P, N;
  void* out;  // [tokens, heads * P]
  int out_dtype;
};

// the sum of x over the GROUPS neighbouring lanes of a value channel (a power of two up to 32)
template <int GROUPS>
__device__ __forceinline__ float lanes_sum(float x) {
#pragma unroll
  for (int offset = 1; offset < GROUPS; offset <<= 1) x += __shfl_xor(x, offset, kWave);
  return x;
}

// The recurrence token by token, for any types and sizes: a block takes one head of one sequence and a slab of value channels;
// a thread keeps 8 states of one channel (two runs of 4), the threads of a channel are neighbouring lanes.  Tokens come
// through LDS a chunk at a time.
template <int GROUPS>
__global__ __launch_bounds__(256) void state_space_scan_kernel(SpaceArgs a) {
  constexpr int kPad = GROUPS * 8, kPer = kWave / GROUPS, kCols = 4 * kPer, kChunk = GROUPS >= 32 ? 16 : 32;
  __shared__ __attribute__((aligned(16))) float bc[kChunk][2][kPad];
  __shared__ float xs[kChunk][kCols];
  __shared__ float step[kChunk][2];  // exp(-rate dt), dt
  const int b = blockIdx.z, head = blockIdx.y;
  const int slot = a.seq_slot[b];
  if (slot < 0) return;
  const int begin = a.seq_start[b], end = a.seq_start[b + 1];
  if (end <= begin) return;
  const int N = a.N, P = a.P, inner = a.heads * P;
  const int group_of = head / (a.heads / a.groups);
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int group = lane % GROUPS, col_in_block = wave * kPer + lane / GROUPS;
  const int col = blockIdx.x * kCols + col_in_block;
  const bool live = col < P;
  float* state = a.state + (((size_t)slot * a.heads + head) * P + (live ? col : 0)) * N;
  int at[8];  // this thread's states
  float S[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    at[r] = (r < 4 ? 0 : kPad / 2) + group * 4 + r % 4;
    S[r] = live && at[r] < N ? state[at[r]] : 0.0f;
  }
  const float D = a.D[head], rate = a.rate[head], dt_bias = a.dt_bias[head];
  for (int t0 = begin; t0 < end; t0 += kChunk) {
    const int count = min(kChunk, end - t0);
    __syncthreads();  // the chunk before has been read
    for (int i = threadIdx.x; i < count * 2 * kPad; i += blockDim.x) {
      const int j = i / (2 * kPad), which = (i / kPad) & 1, n = i % kPad;
      bc[j][which][n] = n < N ? load_as_f32(a.xbc, a.xbc_dtype, (size_t)(t0 + j) * a.xbc_stride + inner + (size_t)which * a.groups * N + (size_t)group_of * N + n) : 0.0f;
    }
    for (int i = threadIdx.x; i < count * kCols; i += blockDim.x) {
      const int j = i / kCols, c = blockIdx.x * kCols + i % kCols;
      xs[j][i % kCols] = c < P ? load_as_f32(a.xbc, a.xbc_dtype, (size_t)(t0 + j) * a.xbc_stride + (size_t)head * P + c) : 0.0f;
    }
    if ((int)threadIdx.x < count) {
      const float dt = softplus_f(load_as_f32(a.dt, a.dt_dtype, (size_t)(t0 + threadIdx.x) * a.dt_stride + head) + dt_bias);
      step[threadIdx.x][0] = expf(-rate * dt);
      step[threadIdx.x][1] = dt;
    }
    __syncthreads();
    for (int j = 0; j < count; ++j) {
      const float keep = step[j][0], x = xs[j][col_in_block], dx = step[j][1] * x;
      const float* B = &bc[j][0][0];
      const float* C = &bc[j][1][0];
      float y = 0.0f;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const float4 b4 = *(const float4*)(B + half * (kPad / 2) + group * 4), c4 = *(const float4*)(C + half * (kPad / 2) + group * 4);
        const float bv[4] = {b4.x, b4.y, b4.z, b4.w}, cv[4] = {c4.x, c4.y, c4.z, c4.w};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          S[4 * half + r] = fmaf(keep, S[4 * half + r], dx * bv[r]);
          y = fmaf(S[4 * half + r], cv[r], y);
        }
      }
      y = lanes_sum<GROUPS>(y);
      if (group == 0 && live) {
        const size_t row = (size_t)(t0 + j);
        const float z = load_as_f32(a.z, a.z_dtype, row * a.z_stride + (size_t)head * P + col);
        store_from_f32(a.out, a.out_dtype, row * inner + (size_t)head * P + col, fmaf(D, x, y) * (z * sigmoid_f(z)));
      }
    }
  }
  if (!live) return;
#pragma unroll
  for (int r = 0; r < 8; ++r)
    if (at[r] < N) state[at[r]] = S[r];
}

// -----------------------------------------------------------------------------
// Prompts of bfloat16 rows, 64 tokens at a time on the matrix cores.  With l_t the sum of -rate dt up to token t of the chunk and S
// the state before it,
//     y_t = e^(l_t) S C_t + sum over s <= t of e^(l_t - l_s) dt_s (C_t . B_s) x_s + D x_t
//     S  <- e^(l_63) S + sum over s of e^(l_63 - l_s) dt_s x_s B_s^T
// B, C and x are bfloat16 as they are; what is 32-bit (the state, the weights of the sums) meets them as two bfloat16 numbers
// whose sum holds 16 bits of it, with 32-bit sums, and the state itself stays in 32-bit registers from chunk to chunk.
//
// A block of 4 waves takes 16 value channels of one head of one sequence and walks its chunks; wave w makes the outputs of tokens
// 16 w .. 16 w + 15 and keeps every fourth tile of 16 states.  NK: N in steps of 32, filled up with zeros.
// -----------------------------------------------------------------------------
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

constexpr int kSpan = 64;    // tokens of a chunk
constexpr int kSlab = 16;    // value channels of a block
constexpr int kTokRow = kSpan + 8;  // bfloat16 of a row along the tokens in LDS

template <int NK>
struct ChunkLds {
  static constexpr int kRow = 32 * NK + 8;
  bf16_t b[kSpan][kRow];         // B, a token a row
  bf16_t bt[32 * NK][kTokRow];   // B, a state a row
  bf16_t xt[kSlab][kTokRow];     // x, a value channel a row
  bf16_t s_hi[kSlab][kRow];      // the state before the chunk, a value channel a row
  bf16_t s_lo[kSlab][kRow];
  float sum[kSpan];              // l_t in powers of two
  float dt[kSpan];
  float weight[kSpan];           // e^(l_63 - l_t) dt_t
};

__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (__bf16)0.0f;
  return z;
}

__device__ __forceinline__ void split_two(const float (&v)[8], bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    hi[i] = (__bf16)v[i];
    lo[i] = (__bf16)(v[i] - (float)hi[i]);
  }
}

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// x from the lane `OFFSET` places before in its row of 16 lanes, 0 where there is none
template <int OFFSET>
__device__ __forceinline__ float from_before(float x) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), 0x110 + OFFSET, 0xF, 0xF, false));
}
__device__ __forceinline__ float lane_value(float x, int lane) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), lane)); }

// ZFOURS: z's rows lie on 8-byte boundaries.  Every load of a chunk is asked for unconditionally and kept as it arrives: a load behind a
// branch, or one that is converted at once, makes the compiler wait for all that were asked for before it.  (States beyond N repeat
// the last ones; C is zero there, so nothing of them reaches an output, and they are not stored.)
template <int NK, bool ZFOURS>
__global__ __launch_bounds__(256) void state_space_chunks_kernel(SpaceArgs a, int slabs, int items) {
  extern __shared__ __attribute__((aligned(16))) char chunk_lds[];
  ChunkLds<NK>& lds = *(ChunkLds<NK>*)chunk_lds;
  constexpr int kItems = NK >= 4 ? NK / 4 : 1;   // (four tokens, eight states) that a thread brings of a chunk's B
  constexpr int kTiles = NK >= 2 ? NK / 2 : 1;   // tiles of 16 states that a wave keeps
  // a die takes neighbouring heads, which share their group's B and C
  int item;
  {
    const int die = blockIdx.x % 8, nth = blockIdx.x / 8, each = items / 8, more = items % 8;
    if (nth >= each + (die < more ? 1 : 0)) return;
    item = die * each + (die < more ? die : more) + nth;
  }
  const int slab = item % slabs, head = item / slabs % a.heads, b = item / slabs / a.heads;
  const int slot = a.seq_slot[b];
  if (slot < 0) return;
  const int begin = a.seq_start[b], end = a.seq_start[b + 1];
  if (end <= begin) return;
  const int N = a.N, P = a.P, inner = a.heads * P;
  const int tid = threadIdx.x, lane = tid % kWave, wave = __builtin_amdgcn_readfirstlane(tid / kWave), r = lane % 16, g = lane / 16;
  const int group_of = head / (a.heads / a.groups);
  const bf16_t* rows = (const bf16_t*)a.xbc;
  const int b_at = inner + group_of * N, c_at = b_at + a.groups * N, x_at = head * P + slab * kSlab;
  const float rate = a.rate[head] * kLog2e, dt_bias = a.dt_bias[head], D = a.D[head];
  float* state = a.state + (((size_t)slot * a.heads + head) * P + slab * kSlab + r) * N;  // of this lane's value channel

  f32x4 S[kTiles];
#pragma unroll
  for (int i = 0; i < kTiles; ++i) {
    const int n = 16 * (wave + 4 * i) + 4 * g;
    S[i] = *(const f32x4*)(state + min(n, N - 4));
  }
  auto keep_state = [&]() {  // the state as the next chunk's products read it
#pragma unroll
    for (int i = 0; i < kTiles; ++i) {
      if (NK == 1 && wave >= 2) continue;
      bf16x4 hi, lo;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        hi[e] = (__bf16)S[i][e];
        lo[e] = (__bf16)(S[i][e] - (float)hi[e]);
      }
      const int n = 16 * (wave + 4 * i) + 4 * g;
      *(bf16x4*)&lds.s_hi[r][n] = hi;
      *(bf16x4*)&lds.s_lo[r][n] = lo;
    }
  };

  // what a chunk brings, asked for while the chunk before is worked on
  // (loads end in the order they were asked for: a number asked for inside a chunk would be waited for behind all of these)
  bf16x8 b_in[kItems][4], c_in[NK], x_in;
  bf16x4 own_in, z_in;
  bf16_t z_one[4], dt_in;
  auto ask = [&](int t0) {
    auto row = [&](int t) { return (size_t)min(t0 + t, end - 1) * a.xbc_stride; };  // (beyond the end: the last again, its weight is zero)
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      const int it = tid + 256 * i, quad = it % 16, piece = it / 16;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        b_in[i][j] = *(const bf16x8*)(rows + row(4 * quad + j) + b_at + min(8 * piece, N - 8));
    }
#pragma unroll
    for (int k = 0; k < NK; ++k) c_in[k] = *(const bf16x8*)(rows + row(16 * wave + r) + c_at + min(32 * k + 8 * g, N - 8));
    x_in = *(const bf16x8*)(rows + row(tid / 2 % kSpan) + x_at + 8 * (tid % 2));
    dt_in = ((const bf16_t*)a.dt)[(size_t)min(t0 + lane, end - 1) * a.dt_stride + head];
    own_in = *(const bf16x4*)(rows + row(16 * wave + r) + x_at + 4 * g);
    const bf16_t* zp = (const bf16_t*)a.z + (size_t)min(t0 + 16 * wave + r, end - 1) * a.z_stride + x_at + 4 * g;
    if constexpr (ZFOURS) {
      z_in = *(const bf16x4*)zp;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) z_one[e] = zp[e];
    }
  };
  ask(begin);
  keep_state();
  for (int t0 = begin; t0 < end; t0 += kSpan) {
    const int count = min(kSpan, end - t0);
    // into LDS (behind the barrier that ended the chunk before)
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      const int it = tid + 256 * i, quad = it % 16, piece = it / 16;
      if (piece < 4 * NK) {
#pragma unroll
        for (int j = 0; j < 4; ++j) *(bf16x8*)&lds.b[4 * quad + j][8 * piece] = b_in[i][j];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const bf16x4 four = {b_in[i][0][e], b_in[i][1][e], b_in[i][2][e], b_in[i][3][e]};
          *(bf16x4*)&lds.bt[8 * piece + e][4 * quad] = four;
        }
      }
    }
    if (tid < 2 * kSpan) {
#pragma unroll
      for (int e = 0; e < 8; ++e) lds.xt[8 * (tid % 2) + e][tid / 2] = x_in[e];
    }
    // lane l: token l's step and the sums of the decays' logarithms (every wave for itself)
    const float dt = lane < count ? softplus_fast((float)dt_in + dt_bias) : 0.0f;
    float sum = -rate * dt;
    sum += from_before<1>(sum);
    sum += from_before<2>(sum);
    sum += from_before<4>(sum);
    sum += from_before<8>(sum);
    {  // (rows of 16 lanes are summed up; the rows before a lane's own)
      const float row0 = lane_value(sum, 15), row1 = row0 + lane_value(sum, 31), row2 = row1 + lane_value(sum, 47);
      sum += g == 0 ? 0.0f : (g == 1 ? row0 : (g == 2 ? row1 : row2));
    }
    const float total = lane_value(sum, kWave - 1);
    if (wave == 0) {
      lds.sum[lane] = sum;
      lds.dt[lane] = dt;
      lds.weight[lane] = exp2_fast(total - sum) * dt;
    }
    bf16x8 c[NK];
#pragma unroll
    for (int k = 0; k < NK; ++k) c[k] = 32 * k + 8 * g < N ? c_in[k] : zero8();
    const bf16x4 own = own_in;
    bf16x4 zv;
#pragma unroll
    for (int e = 0; e < 4; ++e) zv[e] = ZFOURS ? z_in[e] : z_one[e];
    __syncthreads();
    const float my_sum = lds.sum[16 * wave + r];  // of this lane's token
    if (t0 + kSpan < end) ask(t0 + kSpan);
    const int t = 16 * wave + r;
    const bool live = t < count;
    const size_t out_row = (size_t)min(t0 + t, end - 1);
    f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      y = mfma(*(const bf16x8*)&lds.s_hi[r][32 * k + 8 * g], c[k], y);
      y = mfma(*(const bf16x8*)&lds.s_lo[r][32 * k + 8 * g], c[k], y);
    }
    y = y * exp2_fast(my_sum);
    for (int block = 0; block <= wave / 2; ++block) {  // 32 tokens s at a time
      float m[8];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        // (rows in an order that leaves a lane eight tokens one behind the other: row 4 g' + e is token 8 g' + 4 half + e)
        const int s_row = 32 * block + 8 * (r / 4) + 4 * half + r % 4;
        f32x4 dots = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int k = 0; k < NK; ++k) dots = mfma(*(const bf16x8*)&lds.b[s_row][32 * k + 8 * g], c[k], dots);
        const int s0 = 32 * block + 8 * g + 4 * half;
        const f32x4 sums = *(const f32x4*)&lds.sum[s0], dts = *(const f32x4*)&lds.dt[s0];
#pragma unroll
        for (int e = 0; e < 4; ++e) m[4 * half + e] = s0 + e <= t ? dots[e] * dts[e] * exp2_fast(my_sum - sums[e]) : 0.0f;
      }
      bf16x8 hi, lo;
      split_two(m, hi, lo);
      const bf16x8 xv = *(const bf16x8*)&lds.xt[r][32 * block + 8 * g];
      y = mfma(xv, hi, y);
      y = mfma(xv, lo, y);
    }
    if (live) {
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float z = (float)zv[e];
        v[e] = fmaf(D, (float)own[e], y[e]) * (z * sigmoid_f(z));
      }
      const size_t at = out_row * inner + x_at + 4 * g;
      if (a.out_dtype == NNIS_F32) {
        *(f32x4*)((float*)a.out + at) = (f32x4){v[0], v[1], v[2], v[3]};
      } else {
        const bf16x4 four = {(__bf16)v[0], (__bf16)v[1], (__bf16)v[2], (__bf16)v[3]};
        *(bf16x4*)((bf16_t*)a.out + at) = four;
      }
    }
    // the state behind the chunk
    const float keep = exp2_fast(total);
#pragma unroll
    for (int i = 0; i < kTiles; ++i) S[i] = S[i] * keep;
#pragma unroll
    for (int block = 0; block < 2; ++block) {
      const bf16x8 xv = *(const bf16x8*)&lds.xt[r][32 * block + 8 * g];
      const f32x4 w0 = *(const f32x4*)&lds.weight[32 * block + 8 * g], w1 = *(const f32x4*)&lds.weight[32 * block + 8 * g + 4];
      float v[8];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[e] = (float)xv[e] * w0[e];
        v[4 + e] = (float)xv[4 + e] * w1[e];
      }
      bf16x8 hi, lo;
      split_two(v, hi, lo);
#pragma unroll
      for (int i = 0; i < kTiles; ++i) {
        if (NK == 1 && wave >= 2) continue;
        const bf16x8 bv = *(const bf16x8*)&lds.bt[16 * (wave + 4 * i) + r][32 * block + 8 * g];
        S[i] = mfma(bv, hi, S[i]);
        S[i] = mfma(bv, lo, S[i]);
      }
    }
    __syncthreads();  // everything of this chunk has been read
    keep_state();
  }
#pragma unroll
  for (int i = 0; i < kTiles; ++i) {
    const int n = 16 * (wave + 4 * i) + 4 * g;
    if (n < N && wave + 4 * i < 2 * NK) *(f32x4*)(state + n) = S[i];
  }
}

// -----------------------------------------------------------------------------
// A step of single tokens, the convolution included: `rows` are the projection's own, and the inputs before the token come
// from the convolution's state [slots, taps, channels] (position p's in row p % taps: the token's row is one that nobody reads
// in this step; the block that has a channel's first use writes it).  A block takes one head of one sequence and COLS value
// channels; a thread keeps 8 states (two runs of 4) of each of its channels, the GROUPS threads of a channel are neighbouring
// lanes.
// -----------------------------------------------------------------------------
struct StepArgs {
  SpaceArgs a;             // (xbc: the projection's columns before the convolution)
  const float* taps_w;     // [taps, channels]
  const float* conv_bias;  // [channels]
  float* ring;             // [slots, taps, channels]
  const int* tok_pos;
  int taps, channels;
};

template <int GROUPS, int PER>
__global__ __launch_bounds__(256) void state_space_step_kernel(StepArgs s) {
  const SpaceArgs& a = s.a;
  constexpr int kPad = GROUPS * 8, kLanes = 4 * (kWave / GROUPS), kCols = PER * kLanes;
  __shared__ __attribute__((aligned(16))) float bc[2][kPad];
  __shared__ float xs[kCols];
  const int b = blockIdx.z, head = blockIdx.y, col0 = blockIdx.x * kCols;
  const int slot = a.seq_slot[b];
  const int token = a.seq_start[b];
  const int N = a.N, P = a.P, inner = a.heads * P;
  if (slot < 0) return;
  const int per_group = a.heads / a.groups, group_of = head / per_group;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int group = lane % GROUPS, own = wave * (kWave / GROUPS) + lane / GROUPS;
  float* state = a.state + ((size_t)slot * a.heads + head) * P * N;
  f32x4 S[PER][2];
  bool here[2];
#pragma unroll
  for (int h = 0; h < 2; ++h) here[h] = h * (kPad / 2) + group * 4 < N;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int col = min(col0 + i * kLanes + own, P - 1);
#pragma unroll
    for (int h = 0; h < 2; ++h) S[i][h] = here[h] ? *(const f32x4*)(state + (size_t)col * N + h * (kPad / 2) + group * 4) : (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
  }
  const float z_dt = load_as_f32(a.dt, a.dt_dtype, (size_t)token * a.dt_stride + head);
  const int pos = s.tok_pos[token];
  float* ring = s.ring + (size_t)slot * s.taps * s.channels;
  for (int i = threadIdx.x; i < 2 * kPad + kCols; i += blockDim.x) {
    int c = -1;
    bool writes;
    if (i < 2 * kPad) {
      const int which = i / kPad, n = i % kPad;
      if (n < N) c = inner + which * a.groups * N + group_of * N + n;
      writes = head % per_group == 0 && blockIdx.x == 0;
    } else {
      if (col0 + i - 2 * kPad < P) c = head * P + col0 + i - 2 * kPad;
      writes = true;
    }
    float v = 0.0f;
    if (c >= 0) {
      const float now = load_as_f32(a.xbc, a.xbc_dtype, (size_t)token * a.xbc_stride + c);
      v = s.conv_bias[c];
      for (int j = 0; j + 1 < s.taps; ++j) {
        const int at = pos - (s.taps - 1) + j;
        if (at >= 0) v = fmaf(s.taps_w[(size_t)j * s.channels + c], ring[(size_t)(at % s.taps) * s.channels + c], v);
      }
      v = fmaf(s.taps_w[(size_t)(s.taps - 1) * s.channels + c], now, v);
      v = v * sigmoid_f(v);
      if (a.xbc_dtype == NNIS_BF16) v = (float)(bf16_t)v;  // (as prompts leave it)
      if (writes) ring[(size_t)(pos % s.taps) * s.channels + c] = now;
    }
    if (i < 2 * kPad) bc[i / kPad][i % kPad] = v;
    else xs[i - 2 * kPad] = v;
  }
  const float dt = softplus_f(z_dt + a.dt_bias[head]);
  const float keep = expf(-a.rate[head] * dt), D = a.D[head];
  __syncthreads();
  f32x4 B[2], C[2];
#pragma unroll
  for (int h = 0; h < 2; ++h) {
    B[h] = *(const f32x4*)&bc[0][h * (kPad / 2) + group * 4];
    C[h] = *(const f32x4*)&bc[1][h * (kPad / 2) + group * 4];
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int col = col0 + i * kLanes + own;
    const float x = xs[i * kLanes + own], dx = dt * x;
    float y = 0.0f;
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][h][e] = fmaf(keep, S[i][h][e], dx * B[h][e]);
        y = fmaf(S[i][h][e], C[h][e], y);
      }
    y = lanes_sum<GROUPS>(y);
    if (col >= P) continue;
#pragma unroll
    for (int h = 0; h < 2; ++h)
      if (here[h]) *(f32x4*)(state + (size_t)col * N + h * (kPad / 2) + group * 4) = S[i][h];
    if (group == 0) {
      const float z = load_as_f32(a.z, a.z_dtype, (size_t)token * a.z_stride + (size_t)head * P + col);
      store_from_f32(a.out, a.out_dtype, (size_t)token * inner + (size_t)head * P + col, fmaf(D, x, y) * (z * sigmoid_f(z)));
    }
  }
}

// The norm in parts for rows of four channels a thread and access, kept in registers between the two passes: a block a (row, part)
// of up to 4096 channels.
template <typename T>
__global__ __launch_bounds__(256) void parts_norm4_kernel(const T* __restrict__ x, const float* __restrict__ weight, bf16_t* __restrict__ y, int parts,
                                                          int size, float eps) {
  __shared__ float scratch[16];
  constexpr int kKeep = 4;
  const int part = blockIdx.x % parts;
  const size_t base = (size_t)blockIdx.x * size;
  f32x4 v[kKeep], w[kKeep];
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < kKeep; ++i) {
    const int c = 4 * (threadIdx.x + i * blockDim.x);
    if (c < size) {
      if constexpr (sizeof(T) == 4) {
        v[i] = *(const f32x4*)(x + base + c);
      } else {
        const bf16x4 four = *(const bf16x4*)(x + base + c);
        v[i] = (f32x4){(float)four[0], (float)four[1], (float)four[2], (float)four[3]};
      }
      w[i] = *(const f32x4*)(weight + (size_t)part * size + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(v[i][e], v[i][e], ss);
    }
  }
  const float inv = 1.0f / sqrtf((blockDim.x == kWave ? wave_sum(ss) : block_sum(ss, scratch)) / (float)size + eps);
#pragma unroll
  for (int i = 0; i < kKeep; ++i) {
    const int c = 4 * (threadIdx.x + i * blockDim.x);
    if (c < size) {
      bf16x4 out;
#pragma unroll
      for (int e = 0; e < 4; ++e) out[e] = (__bf16)(v[i][e] * inv * w[i][e]);
      *(bf16x4*)(y + base + c) = out;
    }
  }
}

// y[t, part, :] = x / sqrt(mean over the part(x^2) + eps) * weight: a row in `parts` equal parts, each by its own root mean
// square.  A block a (row, part).
__global__ __launch_bounds__(256) void parts_norm_kernel(const void* __restrict__ x, int x_dtype, const float* __restrict__ weight, void* __restrict__ y,
                                                         int y_dtype, int parts, int size, float eps) {
  __shared__ float scratch[16];
  const int part = blockIdx.x % parts;
  const size_t base = (size_t)blockIdx.x * size;
  float ss = 0.0f;
  for (int c = threadIdx.x; c < size; c += blockDim.x) {
    const float v = load_as_f32(x, x_dtype, base + c);
    ss = fmaf(v, v, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)size + eps);
  for (int c = threadIdx.x; c < size; c += blockDim.x)
    store_from_f32(y, y_dtype, base + c, load_as_f32(x, x_dtype, base + c) * inv * weight[(size_t)part * size + c]);
}

}  // namespace

// longest: the most tokens a sequence brings (which kernel runs)
extern "C" int nnis_state_space(const void* xbc, int xbc_dtype, int xbc_stride, const void* dt, int dt_dtype, int dt_stride, const float* rate,
                                const float* dt_bias, const float* D, const void* z, int z_dtype, int z_stride, float* state,
                                const int* seq_slot, const int* seq_start, int batch, int heads, int groups, int P, int N, void* out,
                                int out_dtype, int longest, void* stream) {
  NNIS_REQUIRE(nnis_dtype_ok(xbc_dtype) && nnis_dtype_ok(dt_dtype) && nnis_dtype_ok(z_dtype) && nnis_dtype_ok(out_dtype), "state_space: unknown dtype");
  NNIS_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && P > 0 && N > 0 && N <= 256 && batch >= 0,
               "state_space: bad sizes (%d heads of %d in %d groups, %d states: up to 256 are taken)", heads, P, groups, N);
  NNIS_REQUIRE(xbc_stride >= heads * P + 2 * groups * N && dt_stride >= heads && z_stride >= heads * P, "state_space: rows are too short");
  NNIS_REQUIRE(xbc && dt && rate && dt_bias && D && z && state && seq_slot && seq_start && out, "state_space: a pointer is missing");
  NNIS_REQUIRE(batch <= 65535 && heads <= 65535, "state_space: %d sequences exceed the grid limit", batch);
  if (batch == 0) return 0;
  SpaceArgs a;
  a.xbc = xbc; a.xbc_dtype = xbc_dtype; a.xbc_stride = xbc_stride; a.dt = dt; a.dt_dtype = dt_dtype; a.dt_stride = dt_stride;
  a.rate = rate; a.dt_bias = dt_bias; a.D = D; a.z = z; a.z_dtype = z_dtype; a.z_stride = z_stride; a.state = state;
  a.seq_slot = seq_slot; a.seq_start = seq_start; a.heads = heads; a.groups = groups; a.P = P; a.N = N; a.out = out; a.out_dtype = out_dtype;
  hipStream_t s = (hipStream_t)stream;
  // `longest` tokens or more a sequence, bfloat16 rows on 16-byte boundaries: the matrix cores
  if (longest >= 16 && xbc_dtype == NNIS_BF16 && z_dtype == NNIS_BF16 && dt_dtype == NNIS_BF16 && P % kSlab == 0 && N % 8 == 0 && xbc_stride % 8 == 0 &&
      (uintptr_t)xbc % 16 == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)state % 16 == 0) {
    const bool fours = z_stride % 4 == 0 && (uintptr_t)z % 8 == 0;
    const int slabs = P / kSlab;
    const long long items = (long long)slabs * heads * batch;
    NNIS_REQUIRE(items <= 0x7ffffff0, "state_space: %d sequences exceed the grid limit", batch);
    const dim3 grid((unsigned)((items + 7) / 8 * 8));
    // (beyond 64 KB of LDS a kernel has to be told once; a refusal shows as the launch's failure)
#define NNIS_CHUNKS_OF(NK_, FOURS_)                                                                                            \
  do {                                                                                                                         \
    static const hipError_t allowed = hipFuncSetAttribute((const void*)state_space_chunks_kernel<NK_, FOURS_>,                 \
                                                          hipFuncAttributeMaxDynamicSharedMemorySize, (int)sizeof(ChunkLds<NK_>)); \
    (void)allowed;                                                                                                             \
    hipLaunchKernelGGL((state_space_chunks_kernel<NK_, FOURS_>), grid, dim3(256), sizeof(ChunkLds<NK_>), s, a, slabs, (int)items); \
  } while (0)
#define NNIS_CHUNKS(NK_)                   \
  do {                                     \
    if (fours) NNIS_CHUNKS_OF(NK_, true);  \
    else NNIS_CHUNKS_OF(NK_, false);       \
  } while (0)
    if (N <= 32) NNIS_CHUNKS(1);
    else if (N <= 64) NNIS_CHUNKS(2);
    else if (N <= 128) NNIS_CHUNKS(4);
    else NNIS_CHUNKS(8);
#undef NNIS_CHUNKS
#undef NNIS_CHUNKS_OF
    NNIS_LAUNCH_CHECK("state_space_chunks");
    return 0;
  }
  const int need = (N + 7) / 8;
#define NNIS_SPACE(GROUPS_)                                                                                                          \
  hipLaunchKernelGGL(state_space_scan_kernel<GROUPS_>, dim3((P + 4 * (kWave / GROUPS_) - 1) / (4 * (kWave / GROUPS_)), heads, batch), \
                     dim3(256), 0, s, a)
  if (need <= 1) NNIS_SPACE(1);
  else if (need <= 2) NNIS_SPACE(2);
  else if (need <= 4) NNIS_SPACE(4);
  else if (need <= 8) NNIS_SPACE(8);
  else if (need <= 16) NNIS_SPACE(16);
  else NNIS_SPACE(32);
#undef NNIS_SPACE
  NNIS_LAUNCH_CHECK("state_space");
  return 0;
}

// A step of single tokens with the convolution in it (see StepArgs): N a multiple of 4, taps_w float32 [taps, channels], conv_bias
// float32, ring float32 [slots, taps, channels]
extern "C" int nnis_state_space_step(const void* rows, int rows_dtype, int rows_stride, const void* dt, int dt_dtype, int dt_stride, const float* rate,
                                     const float* dt_bias, const float* D, const void* z, int z_dtype, int z_stride, const float* taps_w,
                                     const float* conv_bias, float* ring, float* state, const int* seq_slot, const int* seq_start,
                                     const int* tok_pos, int batch, int heads, int groups, int P, int N, int taps, void* out, int out_dtype,
                                     void* stream) {
  NNIS_REQUIRE(nnis_dtype_ok(rows_dtype) && nnis_dtype_ok(dt_dtype) && nnis_dtype_ok(z_dtype) && nnis_dtype_ok(out_dtype), "state_space_step: unknown dtype");
  NNIS_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && P > 0 && N > 0 && N <= 256 && N % 4 == 0 && taps > 0 && batch >= 0,
               "state_space_step: bad sizes (%d heads of %d in %d groups, %d states: a multiple of 4 up to 256)", heads, P, groups, N);
  NNIS_REQUIRE(rows_stride >= heads * P + 2 * groups * N && dt_stride >= heads && z_stride >= heads * P, "state_space_step: rows are too short");
  NNIS_REQUIRE(rows && dt && rate && dt_bias && D && z && taps_w && conv_bias && ring && state && seq_slot && seq_start && tok_pos && out,
               "state_space_step: a pointer is missing");
  NNIS_REQUIRE((uintptr_t)state % 16 == 0 && batch <= 65535 && heads <= 65535, "state_space_step: a misaligned state, or %d sequences", batch);
  if (batch == 0) return 0;
  StepArgs t;
  SpaceArgs& a = t.a;
  a.xbc = rows; a.xbc_dtype = rows_dtype; a.xbc_stride = rows_stride; a.dt = dt; a.dt_dtype = dt_dtype; a.dt_stride = dt_stride;
  a.rate = rate; a.dt_bias = dt_bias; a.D = D; a.z = z; a.z_dtype = z_dtype; a.z_stride = z_stride; a.state = state;
  a.seq_slot = seq_slot; a.seq_start = seq_start; a.heads = heads; a.groups = groups; a.P = P; a.N = N; a.out = out; a.out_dtype = out_dtype;
  t.taps_w = taps_w; t.conv_bias = conv_bias; t.ring = ring; t.tok_pos = tok_pos; t.taps = taps; t.channels = heads * P + 2 * groups * N;
  hipStream_t s = (hipStream_t)stream;
  const int need = (N + 7) / 8;
  // value channels a thread takes: more where there are blocks enough for the chip (a block makes its group's B and C anew)
  const bool many = (long long)batch * heads >= 256;
#define NNIS_STEP(GROUPS_)                                                                                              \
  do {                                                                                                                  \
    constexpr int lanes = 4 * (kWave / GROUPS_);                                                                        \
    if (many && P > 2 * lanes)                                                                                          \
      hipLaunchKernelGGL((state_space_step_kernel<GROUPS_, 4>), dim3((P + 4 * lanes - 1) / (4 * lanes), heads, batch), dim3(256), 0, s, t); \
    else if (P > lanes)                                                                                                 \
      hipLaunchKernelGGL((state_space_step_kernel<GROUPS_, 2>), dim3((P + 2 * lanes - 1) / (2 * lanes), heads, batch), dim3(256), 0, s, t); \
    else                                                                                                                \
      hipLaunchKernelGGL((state_space_step_kernel<GROUPS_, 1>), dim3(1, heads, batch), dim3(256), 0, s, t);             \
  } while (0)
  if (need <= 1) NNIS_STEP(1);
  else if (need <= 2) NNIS_STEP(2);
  else if (need <= 4) NNIS_STEP(4);
  else if (need <= 8) NNIS_STEP(8);
  else if (need <= 16) NNIS_STEP(16);
  else NNIS_STEP(32);
#undef NNIS_STEP
  NNIS_LAUNCH_CHECK("state_space_step");
  return 0;
}

extern "C" int nnis_parts_norm(const void* x, int x_dtype, const float* weight, void* y, int y_dtype, int rows, int parts, int size, float eps,
                               void* stream) {
  NNIS_REQUIRE(nnis_dtype_ok(x_dtype) && nnis_dtype_ok(y_dtype), "parts_norm: unknown dtype");
  NNIS_REQUIRE(x && weight && y && rows >= 0 && parts > 0 && size > 0, "parts_norm: bad arguments");
  NNIS_REQUIRE((long long)rows * parts <= 0x7fffffff, "parts_norm: too many rows");
  if (rows == 0) return 0;
  if (y_dtype == NNIS_BF16 && size % 4 == 0 && size <= 4096 && (uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)weight % 16 == 0) {
    const int threads = size <= 1024 ? 64 : 256;
    if (x_dtype == NNIS_F32)
      hipLaunchKernelGGL(parts_norm4_kernel<float>, dim3(rows * parts), dim3(threads), 0, (hipStream_t)stream, (const float*)x, weight, (bf16_t*)y, parts,
                         size, eps);
    else
      hipLaunchKernelGGL(parts_norm4_kernel<bf16_t>, dim3(rows * parts), dim3(threads), 0, (hipStream_t)stream, (const bf16_t*)x, weight, (bf16_t*)y, parts,
                         size, eps);
    NNIS_LAUNCH_CHECK("parts_norm");
    return 0;
  }
  hipLaunchKernelGGL(parts_norm_kernel, dim3(rows * parts), dim3(size >= 512 ? 256 : 64), 0, (hipStream_t)stream, x, x_dtype, weight, y, y_dtype,
                     parts, size, eps);
  NNIS_LAUNCH_CHECK("parts_norm");
  return 0;
}
