// What the files with matrix-core products share: operand and accumulator types, the instruction, stores of four
// consecutive outputs of a token, and the way a product that ends a part of a pre-norm block enters the residual stream.
#pragma once

#include "common.h"

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ bf16x8 load_chunk(const bf16_t* p) { return *(const bf16x8*)p; }

__device__ __forceinline__ bf16x8 zero_chunk() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (__bf16)0.0f;
  return z;
}

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

__device__ __forceinline__ void store4(float* y, size_t index, f32x4 v, int valid, bool vector_ok) {
  if (valid == 4 && vector_ok) {
    *(f32x4*)(y + index) = v;
  } else {
    for (int e = 0; e < valid; ++e) y[index + e] = v[e];
  }
}

__device__ __forceinline__ void store4(bf16_t* y, size_t index, f32x4 v, int valid, bool vector_ok) {
  if (valid == 4 && vector_ok) {
    typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
    bf16x4 packed;
#pragma unroll
    for (int e = 0; e < 4; ++e) packed[e] = (__bf16)v[e];
    *(bf16x4*)(y + index) = packed;
  } else {
    for (int e = 0; e < valid; ++e) y[index + e] = (bf16_t)v[e];
  }
}

// What a projection that ends a part of a pre-norm block does with its result instead of storing it
// (OutT = ResidualOut): the residual stream takes it in, and the norm that follows is prepared.
//   v = resid + y (32-bit, in place);  scaled = bf16(v * gain);  ss[part][token] = sum over the part's
//   columns of v * v.  The norm's 1 / sqrt(mean + eps) is left to the kernel that reads `scaled`: it needs
//   the whole row, and the parts of a row are spread over the blocks.  Statistics as in
//   /root/reference/crates/nnis-model/src/kernels.rs:15-48.
// With `tanh_norms` the block's norms keep no statistics, N(u) = tanh(alpha u) * w + b, and sit on both sides of the sum:
//   v = resid + N_post(y);  scaled = bf16(N_next(v)), the next projection's operand as it is;  ss is written and not read.
// (`gain` is then N_next's weight; all four vectors in gain_dtype.)
struct ResidualOut {
  float* resid;      // [m, n]
  const void* gain;  // [n], the following norm's weight
  int gain_dtype;
  bf16_t* scaled;    // [m, n]
  float* ss;         // [parts, m]; a part is 16 columns (skinny kernel) or a wave's columns (tiled kernel)
  int tanh_norms = 0;
  int tanh_columns = 1;  // n: a flat index's column is index % n
  const void* next_bias = nullptr;
  const void* post_weight = nullptr;
  const void* post_bias = nullptr;
  float next_alpha = 0.0f, post_alpha = 0.0f;
};

// four consecutive columns of a token: what the stream and the gain hold there, asked for early.  A gain in
// bfloat16 stays as it was loaded (two words in g) until it is taken: arithmetic on it here would make the
// kernel wait for the load before its main loop.
struct ResidualHeld {
  f32x4 v, g;
};

__device__ __forceinline__ ResidualHeld residual_ask(const ResidualOut& o, size_t index, int column, int valid, bool vector_ok) {
  ResidualHeld h;
  h.v = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
  h.g = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
  if (valid == 4 && vector_ok) {
    h.v = *(const f32x4*)(o.resid + index);
    if (o.gain_dtype == NNIS_F32) {
      h.g = *(const f32x4*)((const float*)o.gain + column);
    } else {
      const float2 packed = *(const float2*)((const bf16_t*)o.gain + column);
      h.g[0] = packed.x;
      h.g[1] = packed.y;
    }
  } else {
    for (int e = 0; e < valid; ++e) {
      h.v[e] = o.resid[index + e];
      h.g[e] = load_as_f32(o.gain, o.gain_dtype, column + e);
    }
  }
  return h;
}

// tanh by the hardware's exponential and reciprocal, 1 - 2 / (e^(2x) + 1): right at both ends (the power overflows to
// infinity or falls to zero), off by a few 1e-7 in between, which the bfloat16 operand it ends in does not see
__device__ __forceinline__ float tanh_by_exp2(float x) {
  return 1.0f - 2.0f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(x * 2.8853900817779268f) + 1.0f);
}

// four consecutive entries of a vector per column, widened; `whole`: all four exist and lie on an 8- or 16-byte boundary
__device__ __forceinline__ f32x4 four_of(const void* base, int dtype, int column, int valid, bool whole) {
  f32x4 out = {0.0f, 0.0f, 0.0f, 0.0f};
  if (whole) {
    if (dtype == NNIS_F32) return *(const f32x4*)((const float*)base + column);
    const uint2 packed = *(const uint2*)((const bf16_t*)base + column);
    out[0] = __uint_as_float(packed.x << 16);
    out[1] = __uint_as_float(packed.x & 0xffff0000u);
    out[2] = __uint_as_float(packed.y << 16);
    out[3] = __uint_as_float(packed.y & 0xffff0000u);
    return out;
  }
  for (int e = 0; e < valid; ++e) out[e] = load_as_f32(base, dtype, column + e);
  return out;
}

// ... and the lane's accumulator acc taken in; returns the lane's part of the row's sum of squares
__device__ __forceinline__ float residual_take(const ResidualOut& o, const ResidualHeld& h, size_t index, f32x4 acc, int valid,
                                               bool vector_ok) {
  typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
  float sq = 0.0f;
  f32x4 v = h.v, gain = h.g;
  if (valid == 4 && vector_ok && o.gain_dtype != NNIS_F32) {  // four bfloat16 in two words: a float's upper half each
    const unsigned lo = __float_as_uint(h.g[0]), hi = __float_as_uint(h.g[1]);
    gain[0] = __uint_as_float(lo << 16);
    gain[1] = __uint_as_float(lo & 0xffff0000u);
    gain[2] = __uint_as_float(hi << 16);
    gain[3] = __uint_as_float(hi & 0xffff0000u);
  }
  bf16x4 scaled;
  if (o.tanh_norms) {
    // (the three other vectors are asked for here, behind the main loop: a few words that the caches hold)
    const int column = (int)(index % (size_t)o.tanh_columns);
    const bool whole = valid == 4 && vector_ok;
    const f32x4 post_w = four_of(o.post_weight, o.gain_dtype, column, valid, whole);
    const f32x4 post_b = four_of(o.post_bias, o.gain_dtype, column, valid, whole);
    const f32x4 next_b = four_of(o.next_bias, o.gain_dtype, column, valid, whole);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[e] += tanh_by_exp2(o.post_alpha * acc[e]) * post_w[e] + post_b[e];
      scaled[e] = (__bf16)(tanh_by_exp2(o.next_alpha * v[e]) * gain[e] + next_b[e]);
    }
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[e] += acc[e];
      if (e < valid) sq = fmaf(v[e], v[e], sq);
      scaled[e] = (__bf16)(v[e] * gain[e]);
    }
  }
  if (valid == 4 && vector_ok) {
    *(f32x4*)(o.resid + index) = v;
    *(bf16x4*)(o.scaled + index) = scaled;
  } else {
    for (int e = 0; e < valid; ++e) {
      o.resid[index + e] = v[e];
      o.scaled[index + e] = scaled[e];
    }
  }
  return sq;
}

struct PairScratch {
  float* sums;  // [strips][2][MT][64 lanes][4]
  int* count;   // [strips], zero between calls
};

// Where two blocks that share a strip meet, called by the one wave of either that is left with the block's sums: true for
// the second, whose acc then holds both blocks' sums; false for the first, which is done.
template <int MT>
__device__ __forceinline__ bool pair_meets(f32x4 (&acc)[MT], const PairScratch& pair, int strip, int which, int lane) {
  // The sums go out past the caches, are waited for, and then the count:
  // who finds it at one has the other block's sums in memory.  All of it with relaxed order at agent scope,
  // which rests on three facts of this chip and not on the language's memory model: (1) a wave's stores are
  // counted by vmcnt, and `s_waitcnt vmcnt(0)` below ends only when they have been written where agent-scope
  // accesses see them; (2) atomic loads and stores at agent scope go past the dies' own L2 (each die has
  // one), so the second block reads what the first wrote and not a line its die had kept; (3) a wave issues
  // no load before the branch it stands behind is decided, so the sums are not read before the count.  The
  // same with a release on the count and an acquire fence for the second block (the compiler then writes
  // back and invalidates the L2 around them) was measured: 2048 x 5632 at 1 / 8 / 16 tokens 7.8 / 8.3 / 9.7
  // -> 10.1 / 10.4 / 12.0 us, 2048 x 8192 9.7 / 10.2 / 11.7 -> 12.4 / 13.3 / 15.2: more than the second
  // block gains.  The asm statements keep the compiler from moving memory accesses across them.
  float* mine = pair.sums + ((size_t)strip * 2 + which) * (MT * kWave * 4);
  const float* theirs = pair.sums + ((size_t)strip * 2 + 1 - which) * (MT * kWave * 4);
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      __hip_atomic_store(mine + (t * kWave + lane) * 4 + e, acc[t][e], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  int before = 0;
  if (lane == 0) before = __hip_atomic_fetch_add(pair.count + strip, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  before = __builtin_amdgcn_readfirstlane(before);
  asm volatile("" ::: "memory");
  if (before == 0) return false;
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      acc[t][e] += __hip_atomic_load(theirs + (t * kWave + lane) * 4 + e, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  if (lane == 0) __hip_atomic_store(pair.count + strip, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  return true;
}

}  // namespace
