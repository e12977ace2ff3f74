// A token's own input to a layer, gated by the stream and normed on its way into it:
//     g = gelu_tanh(W_g x) * e,   e = columns first .. first + dim - 1 of the token's row of a table
//     x += y / sqrt(mean(y^2) + eps) * w_out,   y = W_p g,      and the next sublayer's rows h = x / sqrt(mean(x^2) + eps) * w_in
//
//   token_gate   g from ready-made logits, for any types and sizes
//   token_side   all of it in one kernel, 16 tokens a block: bfloat16 rows and packed weights (common.h), 32-bit sums
#include "common.h"

thread_local char g_nnis_error[512] = {0};
extern "C" const char* nnis_last_error() { return g_nnis_error; }

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ float gelu_tanh_f(float v) {  // (1 + tanh u) / 2 = sigmoid(2 u)
  const float u2 = 1.5957691216057308f * fmaf(0.044715f * v * v, v, v);
  return v / (1.0f + expf(-u2));
}

// out[t, c] = gelu_tanh(z[t, c]) * table[ids[t], first + c]: a layer's gate on the tokens' own input (0 for an id outside the table)
__global__ void token_gate_kernel(const void* __restrict__ z, int z_dtype, const int* __restrict__ ids, const void* __restrict__ table, int table_dtype,
                                  int vocab, int columns, int first, void* __restrict__ out, int out_dtype, int dim, size_t total) {
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (size_t)gridDim.x * blockDim.x) {
    const size_t t = i / dim, c = i % dim;
    const float v = load_as_f32(z, z_dtype, i);
    const float gate = gelu_tanh_f(v);
    const int id = ids[t];
    const bool inside = id >= 0 && id < vocab;  // (padding rows carry -1: nothing is read outside the table)
    store_from_f32(out, out_dtype, i, inside ? gate * load_as_f32(table, table_dtype, (size_t)id * columns + first + c) : 0.0f);
  }
}

struct SideArgs {
  const bf16_t* rows;   // [m, width]: the stream's rows
  const bf16_t* w_gate; // [dim, width], packed
  const bf16_t* w_proj; // [width, dim], packed
  const int* ids;       // [m]
  const bf16_t* table;  // [vocab, columns]
  int vocab, columns, first, dim;
  float* x;             // [m, width]: the stream
  const float* w_out;   // [width]
  const float* w_in;    // [width] or null (then no rows out)
  bf16_t* h;            // [m, width]
  float eps;
  int m, width;
};

constexpr int kWaves = 8;

// STRIPS: strips of 16 gate outputs; OUT: strips of 16 channels of the stream that a wave takes.
// The gate's product deals K to the waves, each with all of the strips; the other product deals its strips.  Both leave a lane
// four consecutive outputs of one token.
template <int STRIPS, int OUT>
__global__ __launch_bounds__(64 * kWaves) void token_side_kernel(SideArgs a) {
  extern __shared__ __attribute__((aligned(16))) char side_lds[];
  constexpr int kChunks = (STRIPS + 3) / 4;       // of 64 k of the second product
  constexpr int kRow = 64 * kChunks + 8;
  f32x4* part = (f32x4*)side_lds;                 // [wave][strip][lane]
  bf16_t* gs = (bf16_t*)(part + kWaves * STRIPS * kWave);  // [16 tokens][kRow]
  __shared__ float squares[2][kWaves][16];
  const int lane = threadIdx.x % kWave, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), r = lane % 16, g = lane / 16;
  const int row0 = blockIdx.x * 16, row = min(row0 + r, a.m - 1);
  const bool live = row0 + r < a.m;
  const int K = a.width;
  {
    f32x4 acc[STRIPS];
#pragma unroll
    for (int s = 0; s < STRIPS; ++s) acc[s] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    const bf16_t* x_row = a.rows + (size_t)row * K + 16 * g;
    const bf16_t* w = a.w_gate + nnis_packed_lane(r, g, K);
    const size_t strip = nnis_packed_strip_elems(K);
    const int strips = (a.dim + 15) / 16, chunks = nnis_packed_chunks(K);
#pragma unroll 2
    for (int c = wave; c < chunks; c += kWaves) {
      bf16x8 xv[2], wv[STRIPS][2];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const bool inside = 64 * c + 16 * g + 8 * half < K;  // (a multiple of 16: a run of 8 is inside or not; beyond, the weights are zero)
        xv[half] = *(const bf16x8*)(x_row + (inside ? 64 * c + 8 * half : -16 * g));
#pragma unroll
        for (int s = 0; s < STRIPS; ++s)
          wv[s][half] = *(const bf16x8*)(w + min(s, strips - 1) * strip + (size_t)c * kPackedChunkElems + half * kPackedHalfElems);
      }
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int s = 0; s < STRIPS; ++s) acc[s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[s][half], xv[half], acc[s], 0, 0, 0);
    }
#pragma unroll
    for (int s = 0; s < STRIPS; ++s) part[((size_t)wave * STRIPS + s) * kWave + lane] = acc[s];
  }
  __syncthreads();
  // the gate: a wave a strip at a time
  for (int s = wave; s < 4 * kChunks; s += kWaves) {
    bf16x4 out = {(__bf16)0.0f, (__bf16)0.0f, (__bf16)0.0f, (__bf16)0.0f};
    if (s < STRIPS) {
      f32x4 z = part[(size_t)s * kWave + lane];
#pragma unroll
      for (int w = 1; w < kWaves; ++w) z += part[((size_t)w * STRIPS + s) * kWave + lane];
      const int id = a.ids[row], n = 16 * s + 4 * g;
      if (id >= 0 && id < a.vocab) {  // (padding rows carry -1: nothing is read outside the table)
        const bf16_t* e_row = a.table + (size_t)id * a.columns + a.first + n;
#pragma unroll
        for (int e = 0; e < 4; ++e) out[e] = n + e < a.dim ? (__bf16)(gelu_tanh_f(z[e]) * (float)e_row[e]) : (__bf16)0.0f;
      }
    }
    *(bf16x4*)(gs + (size_t)r * kRow + 16 * s + 4 * g) = out;
  }
  __syncthreads();
  const int n_first = wave * OUT * 16;  // this wave's channels
  f32x4 y[OUT];
  {
    bf16x8 gv[kChunks][2];
#pragma unroll
    for (int c = 0; c < kChunks; ++c)
#pragma unroll
      for (int half = 0; half < 2; ++half) gv[c][half] = *(const bf16x8*)(gs + (size_t)r * kRow + 64 * c + 16 * g + 8 * half);
    const int k_chunks = nnis_packed_chunks(a.dim);  // (a strip may be shorter than this kernel's: its last chunk again, times zeros)
#pragma unroll
    for (int i = 0; i < OUT; ++i) {
      y[i] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
      const int n = min(n_first + 16 * i, K - 16);
      const bf16_t* w = a.w_proj + nnis_packed_lane(n + r, g, a.dim);
#pragma unroll
      for (int c = 0; c < kChunks; ++c)
#pragma unroll
        for (int half = 0; half < 2; ++half)
          y[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(w + (size_t)min(c, k_chunks - 1) * kPackedChunkElems + half * kPackedHalfElems),
                                                         gv[c][half], y[i], 0, 0, 0);
    }
  }
  // the norm on the way out, the sum, the norm on the way in
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < OUT; ++i)
    if (n_first + 16 * i < K) {
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(y[i][e], y[i][e], ss);
    }
  auto over_block = [&](float v, int which) {  // the row's sum: this lane's token over its four lanes and the waves
    v += __shfl_xor(v, 16, kWave);
    v += __shfl_xor(v, 32, kWave);
    if (g == 0) squares[which][wave][r] = v;
    __syncthreads();
    float total = 0.0f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) total += squares[which][w][r];
    return total;
  };
  const float inv = 1.0f / sqrtf(over_block(ss, 0) / (float)K + a.eps);
  float* x_row = a.x + (size_t)row * K;
  float ss2 = 0.0f;
#pragma unroll
  for (int i = 0; i < OUT; ++i) {
    const int n = n_first + 16 * i + 4 * g;
    if (n_first + 16 * i < K) {
      const f32x4 v = *(const f32x4*)(x_row + n), w = *(const f32x4*)(a.w_out + n);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        y[i][e] = fmaf(y[i][e] * inv, w[e], v[e]);
        ss2 = fmaf(y[i][e], y[i][e], ss2);
      }
      if (live) *(f32x4*)(x_row + n) = y[i];
    }
  }
  if (a.h == nullptr) return;
  const float inv2 = 1.0f / sqrtf(over_block(ss2, 1) / (float)K + a.eps);
#pragma unroll
  for (int i = 0; i < OUT; ++i) {
    const int n = n_first + 16 * i + 4 * g;
    if (n_first + 16 * i < K && live) {
      const f32x4 w = *(const f32x4*)(a.w_in + n);
      bf16x4 out;
#pragma unroll
      for (int e = 0; e < 4; ++e) out[e] = (__bf16)(y[i][e] * inv2 * w[e]);
      *(bf16x4*)(a.h + (size_t)row * K + n) = out;
    }
  }
}

}  // namespace

extern "C" int nnis_token_gate(const void* z, int z_dtype, const int* ids, const void* table, int table_dtype, int vocab, int columns, int first,
                               void* out, int out_dtype, int rows, int dim, void* stream) {
  NNIS_REQUIRE(z && ids && table && out && dim > 0 && first >= 0 && first + dim <= columns && vocab > 0, "token_gate: bad arguments");
  NNIS_REQUIRE(nnis_dtype_ok(z_dtype) && nnis_dtype_ok(table_dtype) && nnis_dtype_ok(out_dtype), "token_gate: unknown dtype");
  if (rows <= 0) return 0;
  const size_t total = (size_t)rows * dim;
  const size_t blocks = (total + 255) / 256;
  hipLaunchKernelGGL(token_gate_kernel, dim3((unsigned)(blocks > 65536 ? 65536 : blocks)), dim3(256), 0, (hipStream_t)stream, z, z_dtype, ids, table,
                     table_dtype, vocab, columns, first, out, out_dtype, dim, total);
  NNIS_LAUNCH_CHECK("token_gate");
  return 0;
}

// w_gate, w_proj: packed bfloat16 weights; w_out, w_in: float32; x: the stream, in place; h (with w_in): the next rows, or null
extern "C" int nnis_token_side(const void* rows, const void* w_gate, const void* w_proj, const int* ids, const void* table, int vocab, int columns,
                               int first, int dim, float* x, const float* w_out, const float* w_in, void* h, float eps, int m, int width, void* stream) {
  NNIS_REQUIRE(rows && w_gate && w_proj && ids && table && x && w_out && (h == nullptr) == (w_in == nullptr), "token_side: missing operand");
  NNIS_REQUIRE(dim > 0 && dim % 8 == 0 && dim <= 256 && first >= 0 && first + dim <= columns && vocab > 0 && width > 0 && width % 16 == 0 && width <= 4096,
               "token_side: inputs of a multiple of 8 channels up to 256 for a stream of a multiple of 16 up to 4096, got %d and %d", dim, width);
  for (const void* p : {rows, w_gate, w_proj, (const void*)x, (const void*)w_out, (const void*)w_in, (const void*)h})
    NNIS_REQUIRE((uintptr_t)p % 16 == 0, "token_side: operands must be 16-byte aligned");
  if (m <= 0) return 0;
  const SideArgs a = {(const bf16_t*)rows, (const bf16_t*)w_gate, (const bf16_t*)w_proj, ids, (const bf16_t*)table, vocab, columns, first, dim, x,
                      w_out, w_in, (bf16_t*)h, eps, m, width};
  hipStream_t s = (hipStream_t)stream;
  // (beyond 64 KB of LDS a kernel has to be told once; a refusal shows as the launch's failure)
#define NNIS_SIDE(STRIPS_, OUT_)                                                                                                        \
  do {                                                                                                                                  \
    constexpr int bytes = kWaves * STRIPS_ * kWave * 16 + 16 * (64 * ((STRIPS_ + 3) / 4) + 8) * 2;                                      \
    static const hipError_t allowed = hipFuncSetAttribute((const void*)token_side_kernel<STRIPS_, OUT_>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes); \
    (void)allowed;                                                                                                                      \
    hipLaunchKernelGGL((token_side_kernel<STRIPS_, OUT_>), dim3((m + 15) / 16), dim3(64 * kWaves), bytes, s, a);                        \
  } while (0)
#define NNIS_SIDE_OUT(STRIPS_)                  \
  do {                                          \
    if (width <= 512) NNIS_SIDE(STRIPS_, 4);    \
    else if (width <= 1024) NNIS_SIDE(STRIPS_, 8);   \
    else if (width <= 2048) NNIS_SIDE(STRIPS_, 16);  \
    else NNIS_SIDE(STRIPS_, 32);                \
  } while (0)
  if (dim <= 32) NNIS_SIDE_OUT(2);
  else if (dim <= 64) NNIS_SIDE_OUT(4);
  else if (dim <= 128) NNIS_SIDE_OUT(8);
  else NNIS_SIDE_OUT(16);
#undef NNIS_SIDE_OUT
#undef NNIS_SIDE
  NNIS_LAUNCH_CHECK("token_side");
  return 0;
}
