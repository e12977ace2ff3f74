// Mamba-2's mixer between its projections (state-space duality): a matrix state per head that one number a head and token
// lets decay, and the gated norm in parts behind it.
//
// Rows.  A step's rows are packed: sequence b owns rows seq_start[b] .. seq_start[b + 1] - 1, which continue the sequence in
// slot seq_slot[b] (negative: padding).  `xbc` [tokens, stride] holds, behind the convolution, a token's x (heads * P channels),
// B and C (groups * N each); head h uses group h / (heads / groups).  Per head, S [P, N] (32-bit, column by column of the
// design's [N, P]: a value channel's N states are consecutive) and
//     dt = softplus(z_dt + dt_bias),  S <- exp(-rate dt) S + dt x B^T,  y = S C + D x,   rate = exp(A_log) ready-made
// Decays, step sizes, exponentials, state and sums are 32-bit whatever the storage type.
#include "common.h"

thread_local char g_nnis_error[512] = {0};
extern "C" const char* nnis_last_error() { return g_nnis_error; }

namespace {

constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + exp2_fast(-z * kLog2e)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

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

extern "C" int nnis_state_space(const void* xbc, int xbc_dtype, int xbc_stride, const void* dt, int dt_dtype, int dt_stride, const float* rate,
                                const float* dt_bias, const float* D, const void* z, int z_dtype, int z_stride, float* state,
                                const int* seq_slot, const int* seq_start, int batch, int heads, int groups, int P, int N, void* out,
                                int out_dtype, void* stream) {
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

extern "C" int nnis_parts_norm(const void* x, int x_dtype, const float* weight, void* y, int y_dtype, int rows, int parts, int size, float eps,
                               void* stream) {
  NNIS_REQUIRE(nnis_dtype_ok(x_dtype) && nnis_dtype_ok(y_dtype), "parts_norm: unknown dtype");
  NNIS_REQUIRE(x && weight && y && rows >= 0 && parts > 0 && size > 0, "parts_norm: bad arguments");
  NNIS_REQUIRE((long long)rows * parts <= 0x7fffffff, "parts_norm: too many rows");
  if (rows == 0) return 0;
  hipLaunchKernelGGL(parts_norm_kernel, dim3(rows * parts), dim3(size >= 512 ? 256 : 64), 0, (hipStream_t)stream, x, x_dtype, weight, y, y_dtype,
                     parts, size, eps);
  NNIS_LAUNCH_CHECK("parts_norm");
  return 0;
}
