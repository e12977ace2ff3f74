// A token's own input to a layer, gated by the stream: g = gelu_tanh(W x) * e, e = columns first .. first + dim - 1 of the token's row
// of a table.
//
//   token_gate       g from ready-made logits, for any types and sizes
//   token_gate_rows  the product included: bfloat16 rows and packed weights (common.h), 32-bit sums
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

struct GateArgs {
  const bf16_t* rows;   // [m, width]: the stream's rows
  const bf16_t* w;      // [dim, width], packed
  const int* ids;       // [m]
  const bf16_t* table;  // [vocab, columns]
  int vocab, columns, first, dim;
  bf16_t* out;          // [m, dim]
  int m, width;
};

constexpr int kWaves = 8;

// The gate's product included: a block takes a strip of 16 outputs of 16 tokens, K dealt to its waves.  (The strips of a tile of
// tokens lie side by side: they read the same rows.)
__global__ __launch_bounds__(64 * kWaves) void token_gate_rows_kernel(GateArgs a) {
  __shared__ f32x4 part[kWaves][kWave];
  const int lane = threadIdx.x % kWave, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), r = lane % 16, g = lane / 16;
  const int row = min((int)blockIdx.y * 16 + r, a.m - 1), K = a.width;
  const bf16_t* x_row = a.rows + (size_t)row * K + 16 * g;
  const bf16_t* w = a.w + nnis_packed_lane(16 * blockIdx.x + r, g, K);
  const int n = 16 * blockIdx.x + 4 * g, id = a.ids[row];
  f32x4 z = {0.0f, 0.0f, 0.0f, 0.0f};
  const int chunks = nnis_packed_chunks(K);
  constexpr int kDepth = 4;
  for (int c0 = wave; c0 < chunks; c0 += kWaves * kDepth) {
    bf16x8 xv[kDepth][2], wv[kDepth][2];
#pragma unroll
    for (int d = 0; d < kDepth; ++d)
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int c = c0 + d * kWaves;
        const bool inside = c < chunks && 64 * c + 16 * g + 8 * half < K;
        xv[d][half] = *(const bf16x8*)(x_row + (inside ? 64 * c + 8 * half : -16 * g));
        wv[d][half] = *(const bf16x8*)(w + (size_t)min(c, chunks - 1) * kPackedChunkElems + half * kPackedHalfElems);
        if (!inside) {
#pragma unroll
          for (int e = 0; e < 8; ++e) xv[d][half][e] = (__bf16)0.0f;
        }
      }
#pragma unroll
    for (int d = 0; d < kDepth; ++d)
#pragma unroll
      for (int half = 0; half < 2; ++half) z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[d][half], xv[d][half], z, 0, 0, 0);
  }
  bf16x4 e_own = {(__bf16)0.0f, (__bf16)0.0f, (__bf16)0.0f, (__bf16)0.0f};
  if (wave == 0 && id >= 0 && id < a.vocab) {
    const bf16_t* e_row = a.table + (size_t)id * a.columns + a.first + n;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (n + e < a.dim) e_own[e] = e_row[e];
  }
  part[wave][lane] = z;
  __syncthreads();
  if (wave != 0) return;
#pragma unroll
  for (int o = 1; o < kWaves; ++o) z += part[o][lane];
  if ((int)blockIdx.y * 16 + r >= a.m) return;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (n + e < a.dim) a.out[(size_t)row * a.dim + n + e] = (__bf16)(gelu_tanh_f(z[e]) * (float)e_own[e]);
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

// rows bfloat16 [m, width], w_gate packed [dim, width], table bfloat16 [vocab, columns], out bfloat16 [m, dim]
extern "C" int nnis_token_gate_rows(const void* rows, const void* w_gate, const int* ids, const void* table, int vocab, int columns, int first, int dim,
                                   void* out, int m, int width, void* stream) {
  NNIS_REQUIRE(rows && w_gate && ids && table && out, "token_gate_rows: missing operand");
  NNIS_REQUIRE(dim > 0 && first >= 0 && first + dim <= columns && vocab > 0 && width > 0 && width % 8 == 0, "token_gate_rows: bad sizes (%d from %d of %d, width %d)",
               dim, first, columns, width);
  NNIS_REQUIRE((uintptr_t)rows % 16 == 0 && (uintptr_t)w_gate % 16 == 0, "token_gate_rows: operands must be 16-byte aligned");
  NNIS_REQUIRE((m + 15) / 16 <= 65535, "token_gate_rows: %d rows exceed the grid limit", m);
  if (m <= 0) return 0;
  const GateArgs a = {(const bf16_t*)rows, (const bf16_t*)w_gate, ids, (const bf16_t*)table, vocab, columns, first, dim, (bf16_t*)out, m, width};
  hipLaunchKernelGGL(token_gate_rows_kernel, dim3((dim + 15) / 16, (m + 15) / 16), dim3(64 * kWaves), 0, (hipStream_t)stream, a);
  NNIS_LAUNCH_CHECK("token_gate_rows");
  return 0;
}
