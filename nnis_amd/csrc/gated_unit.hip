// Griffin's real-gated linear recurrent unit between its projections.  Per channel c of token t, with u behind the convolution, the
// channels in `blocks` equal parts of which each has two square maps,
//     zr = R_b u_b,  zi = I_b u_b,  log a = -8 sigmoid(zr + br) rate,   rate = softplus(lam) ready-made
//     S <- a S + sqrt(1 - a^2) sigmoid(zi + bi) u,   out = S * gelu_tanh(y + by)
// A step's rows are packed: sequence b owns rows seq_start[b] .. seq_start[b + 1] - 1, which continue the sequence in slot
// seq_slot[b] (negative: padding); state [slots, width] in 32-bit.  Everything behind u is 32-bit whatever the storage type (the
// maps multiply u and weights as they are stored, with 32-bit sums).
//
// Three kernels: rg_lru_kernel, the recurrence alone behind ready-made logits, for any types and sizes; rg_lru_chunks_kernel, prompts
// of bfloat16 rows, maps and recurrence 128 tokens at a time; rg_lru_step_kernel, single tokens, the convolution included.
#include "common.h"

thread_local char g_nnis_error[512] = {0};
extern "C" const char* nnis_last_error() { return g_nnis_error; }

namespace {

constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + exp2_fast(-z * kLog2e)); }

// -----------------------------------------------------------------------------
// The real-gated linear recurrent unit's recurrence.  Per channel c of row t, with the gates' logits zr and zi:
//     log a = -8 sigmoid(zr + br) rate,   rate = softplus(lam) ready-made
//     S <- a S + sqrt(1 - a^2) sigmoid(zi + bi) u,   out = S * gelu_tanh(y + by)
// over each sequence's rows, from and into state [slots, width] (32-bit).  logits [tokens, blocks, 2, width / blocks]: a
// block's zr, then its zi.  A thread a channel; a long run is cut into pieces as the minGRU's.
// -----------------------------------------------------------------------------
struct UnitArgs {
  const float* logits;
  const float* r_bias;
  const float* i_bias;
  const float* rate;
  const void* u;  // [tokens, u_stride]
  int u_dtype, u_stride;
  const void* y;  // [tokens, y_stride]
  int y_dtype, y_stride;
  const float* y_bias;
  float* state;
  const int* seq_slot;
  const int* seq_start;
  int batch, width, block;  // block: channels of one of the gates' maps
  void* out;
  int out_dtype;
  int piece, pieces;
  float* decay;  // [batch, pieces, width]: a piece's sum of log a
  float* ends;   // [batch, pieces, width]: a piece's end state from zero
};

__device__ __forceinline__ float gelu_tanh_f(float z) {
  const float t = 0.7978845608028654f * fmaf(0.044715f * z * z, z, z);
  return z * sigmoid_f(2.0f * t);  // (1 + tanh t) / 2 = sigmoid(2 t)
}

template <int PASS>
__global__ __launch_bounds__(256) void rg_lru_kernel(UnitArgs a) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int b = blockIdx.y / a.pieces, piece = blockIdx.y % a.pieces;
  const int slot = a.seq_slot[b];
  if (slot < 0 || c >= a.width) return;
  const int start = a.seq_start[b], stop = a.seq_start[b + 1];
  int first = start, last = stop;
  if (a.pieces > 1) {
    first = start + piece * a.piece;
    last = min(stop, first + a.piece);
    if (first >= stop) return;
    if (PASS == 1 && last == stop && piece > 0) return;
  }
  const float br = a.r_bias[c], bi = a.i_bias[c], by = a.y_bias ? a.y_bias[c] : 0.0f, rate = -8.0f * a.rate[c];
  const size_t gate_at = (size_t)(c / a.block) * 2 * a.block + c % a.block;
  float s = 0.0f, logs = 0.0f;
  const size_t mine = ((size_t)b * a.pieces + piece) * a.width + c;
  if (a.pieces == 1) {
    s = a.state[(size_t)slot * a.width + c];
  } else if (PASS == 1) {
    if (piece == 0) a.decay[mine] = s = a.state[(size_t)slot * a.width + c];  // (a copy of the state: see the minGRU)
  } else if (piece == 0) {
    s = a.decay[mine];
  } else {
    s = a.ends[(size_t)b * a.pieces * a.width + c];
#pragma unroll 8
    for (int k = 1; k < piece; ++k) {
      const size_t at = ((size_t)b * a.pieces + k) * a.width + c;
      s = fmaf(expf(a.decay[at]), s, a.ends[at]);
    }
  }
#pragma unroll 4
  for (int t = first; t < last; ++t) {
    const float zr = a.logits[(size_t)t * 2 * a.width + gate_at] + br;
    const float zi = a.logits[(size_t)t * 2 * a.width + gate_at + a.block] + bi;
    const float u = load_as_f32(a.u, a.u_dtype, (size_t)t * a.u_stride + c);
    const float log_a = rate / (1.0f + expf(-zr));
    const float keep = expf(log_a);
    s = fmaf(keep, s, sqrtf(-expm1f(2.0f * log_a)) * (u / (1.0f + expf(-zi))));
    if (PASS == 1) {
      logs += log_a;
    } else {
      const float y = load_as_f32(a.y, a.y_dtype, (size_t)t * a.y_stride + c) + by;
      store_from_f32(a.out, a.out_dtype, (size_t)t * a.width + c, s * gelu_tanh_f(y));
    }
  }
  if (PASS == 1) {
    if (piece > 0) a.decay[mine] = logs;
    a.ends[mine] = s;
  } else if (last == stop) {
    a.state[(size_t)slot * a.width + c] = s;
  }
}


// a token's decay and what it adds, from its logits (biases taken in) and u: log a = rate8 sigmoid(zr), rate8 = -8 rate
struct Decay {
  float keep, add;
};
__device__ __forceinline__ Decay unit_terms(float zr, float zi, float u, float rate8) {
  const float log_a = rate8 * sigmoid_f(zr);
  // 1 - a^2 = -(e^(2 log a) - 1): by its series where a is near one, where 1 - a^2 would round it away
  const float x = 2.0f * log_a;
  const float near = -x * fmaf(x, fmaf(x, fmaf(x, 1.0f / 24.0f, 1.0f / 6.0f), 0.5f), 1.0f);
  const float square = x > -0.05f ? near : 1.0f - exp2_fast(x * kLog2e);
  return {exp2_fast(log_a * kLog2e), __builtin_amdgcn_sqrtf(square) * sigmoid_f(zi) * u};
}

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;
__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (__bf16)0.0f;
  return z;
}

// x from the lane `OFFSET` places before in its row of 16 lanes, `other` where there is none
template <int OFFSET>
__device__ __forceinline__ float from_before(float x, float other) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, other), __builtin_bit_cast(int, x), 0x110 + OFFSET, 0xF, 0xF, false));
}

// Prompts.  A block of 8 waves takes 16 channels of a part and walks its sequence 128 tokens at a time: wave w the tokens 16 w .. 16 w
// + 15, a lane 4 channels of one token (the matrix product's layout: columns are tokens).  The 16 channels' rows of both maps stay
// in registers.  The recurrence is a scan of (keep, add) pairs: over the 16 tokens of a wave by moves between lanes, over the waves
// through LDS.  KB: a part's channels in steps of 32, filled up with zeros.
struct MapArgs {
  UnitArgs a;
  const bf16_t* maps;  // [blocks, 2 * block, block]: a part's R rows, then its I rows
};

constexpr int kWaves = 8, kTokens = 16 * kWaves;

template <int KB>
__global__ __launch_bounds__(64 * kWaves) void rg_lru_chunks_kernel(MapArgs m, int tiles, int items) {
  const UnitArgs& a = m.a;
  __shared__ __attribute__((aligned(16))) float ends[2][kWaves][2][16];  // [chunk's parity][wave][keep, add][channel]
  int item;
  {
    const int die = blockIdx.x % 8, nth = blockIdx.x / 8, each = items / 8, more = items % 8;  // a die takes the tiles of neighbouring parts
    if (nth >= each + (die < more ? 1 : 0)) return;
    item = die * each + (die < more ? die : more) + nth;
  }
  const int blocks = a.width / a.block;
  const int tile = item % tiles, part = item / tiles % blocks, b = item / tiles / blocks;
  const int slot = a.seq_slot[b];
  if (slot < 0) return;
  const int begin = a.seq_start[b], end = a.seq_start[b + 1];
  if (end <= begin) return;
  const int lane = threadIdx.x % kWave, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), r = lane % 16, g = lane / 16;
  const int K = a.block;
  bf16x8 wr[KB], wi[KB];
  {
    const int row = min(16 * tile + r, K - 1);  // (rows beyond the part: not stored)
    const bf16_t* base = m.maps + ((size_t)part * 2 * K + row) * K + 8 * g;
#pragma unroll
    for (int k = 0; k < KB; ++k) {
      const bool inside = 32 * k + 8 * g < K;
      wr[k] = inside ? *(const bf16x8*)(base + 32 * k) : zero8();
      wi[k] = inside ? *(const bf16x8*)(base + (size_t)K * K + 32 * k) : zero8();
    }
  }
  const bool stored = 16 * tile + 4 * g < K;  // (a part is a multiple of 8 channels: this lane's four are inside or not)
  const int c0 = part * K + (stored ? 16 * tile + 4 * g : 0);
  const f32x4 br = *(const f32x4*)(a.r_bias + c0), bi = *(const f32x4*)(a.i_bias + c0), by = *(const f32x4*)(a.y_bias + c0);
  const f32x4 rate8 = *(const f32x4*)(a.rate + c0) * -8.0f;
  f32x4 S = *(const f32x4*)(a.state + (size_t)slot * a.width + c0);
  const bf16_t* u_rows = (const bf16_t*)a.u;
  const bf16_t* y_rows = (const bf16_t*)a.y;
  bf16x8 u_in[KB];
  bf16x4 own_in, y_in;
  auto ask = [&](int t0) {
    const size_t t = min(t0 + 16 * wave + r, end - 1);
    const bf16_t* row = u_rows + t * a.u_stride + (size_t)part * K;
    // (beyond the part: its last channels again, the maps are zero there; no load stands behind a branch)
#pragma unroll
    for (int k = 0; k < KB; ++k) u_in[k] = *(const bf16x8*)(row + min(32 * k + 8 * g, K - 8));
    own_in = *(const bf16x4*)(u_rows + t * a.u_stride + c0);
    y_in = *(const bf16x4*)(y_rows + t * a.y_stride + c0);
  };
  ask(begin);
  int parity = 0;
  for (int t0 = begin; t0 < end; t0 += kTokens, parity ^= 1) {
    f32x4 zr = {0.0f, 0.0f, 0.0f, 0.0f}, zi = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int k = 0; k < KB; ++k) {
      zr = mfma(wr[k], u_in[k], zr);
      zi = mfma(wi[k], u_in[k], zi);
    }
    const bf16x4 own = own_in, yv = y_in;
    const int t = t0 + 16 * wave + r;
    const bool live = t < end;
    if (t0 + kTokens < end) ask(t0 + kTokens);
    float keep[4], add[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const Decay d = unit_terms(zr[e] + br[e], zi[e] + bi[e], (float)own[e], rate8[e]);
      keep[e] = live ? d.keep : 1.0f;
      add[e] = live ? d.add : 0.0f;
    }
    // inclusive scan over the wave's 16 tokens: (k1, a1) then (k2, a2) is (k1 k2, k2 a1 + a2)
#define NNIS_SCAN_STEP(OFFSET_)                                             \
  _Pragma("unroll") for (int e = 0; e < 4; ++e) {                          \
    const float k1 = from_before<OFFSET_>(keep[e], 1.0f), a1 = from_before<OFFSET_>(add[e], 0.0f); \
    add[e] = fmaf(keep[e], a1, add[e]);                                     \
    keep[e] *= k1;                                                          \
  }
    NNIS_SCAN_STEP(1)
    NNIS_SCAN_STEP(2)
    NNIS_SCAN_STEP(4)
    NNIS_SCAN_STEP(8)
#undef NNIS_SCAN_STEP
    if (r == 15) {
      *(f32x4*)&ends[parity][wave][0][4 * g] = (f32x4){keep[0], keep[1], keep[2], keep[3]};
      *(f32x4*)&ends[parity][wave][1][4 * g] = (f32x4){add[0], add[1], add[2], add[3]};
    }
    __syncthreads();  // (the other parity's numbers were read before this barrier's predecessor)
    f32x4 before = S;  // the state before this wave's first token
#pragma unroll
    for (int w = 0; w < kWaves; ++w) {
      const f32x4 k = *(const f32x4*)&ends[parity][w][0][4 * g], ad = *(const f32x4*)&ends[parity][w][1][4 * g];
      if (w == wave) before = S;
#pragma unroll
      for (int e = 0; e < 4; ++e) S[e] = fmaf(k[e], S[e], ad[e]);
    }
    if (live && stored) {
      bf16x4 out;
#pragma unroll
      for (int e = 0; e < 4; ++e) out[e] = (__bf16)(fmaf(keep[e], before[e], add[e]) * gelu_tanh_f((float)yv[e] + by[e]));
      *(bf16x4*)((bf16_t*)a.out + (size_t)t * a.width + c0) = out;
    }
  }
  if (wave == 0 && r == 0 && stored) *(f32x4*)(a.state + (size_t)slot * a.width + c0) = S;
}

// A step of single tokens: a block of 4 waves takes 16 channels of a part for 16 sequences (the product's columns), K dealt to the
// waves.  u is made on the way: x + its bias and the inputs before it, from the convolution's state [slots, taps, width] (position
// p's in row p % taps; the block that owns a channel writes the token's row, which nobody reads in this step).
struct UnitStepArgs {
  MapArgs m;                // (u: the projection's columns of x)
  const float* x_bias;      // [width]
  const float* taps_w;      // [taps, width]
  const float* conv_bias;   // [width]
  float* ring;
  const int* tok_pos;
  int taps;
};

// u of COUNT (4 or 8) channels from c on of the sequence in `slot` at `pos`, as prompts leave it (rounded to bfloat16); now: the inputs
template <int COUNT>
__device__ __forceinline__ void unit_input(const UnitStepArgs& s, int token, int slot, int pos, int c, float (&u)[COUNT], float (&now)[COUNT]) {
  const int width = s.m.a.width;
  const bf16_t* x = (const bf16_t*)s.m.a.u + (size_t)token * s.m.a.u_stride + c;
  const float* ring = s.ring + (size_t)slot * s.taps * width + c;
#pragma unroll
  for (int q = 0; q < COUNT / 4; ++q) {
    const bf16x4 xv = *(const bf16x4*)(x + 4 * q);
    const f32x4 xb = *(const f32x4*)(s.x_bias + c + 4 * q), w = *(const f32x4*)(s.taps_w + (size_t)(s.taps - 1) * width + c + 4 * q);
    f32x4 sum = *(const f32x4*)(s.conv_bias + c + 4 * q);
    for (int j = 0; j + 1 < s.taps; ++j) {
      const int at = pos - (s.taps - 1) + j;
      const f32x4 v = *(const f32x4*)(ring + (size_t)((at + s.taps) % s.taps) * width + 4 * q);  // (before the start: read, not counted)
      const f32x4 wj = *(const f32x4*)(s.taps_w + (size_t)j * width + c + 4 * q);
#pragma unroll
      for (int e = 0; e < 4; ++e) sum[e] = at >= 0 ? fmaf(wj[e], v[e], sum[e]) : sum[e];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      now[4 * q + e] = (float)xv[e] + xb[e];
      u[4 * q + e] = (float)(__bf16)fmaf(w[e], now[4 * q + e], sum[e]);
    }
  }
}

__global__ __launch_bounds__(256) void rg_lru_step_kernel(UnitStepArgs s) {
  const UnitArgs& a = s.m.a;
  __shared__ __attribute__((aligned(16))) float partial[4][2][kWave][4];
  const int K = a.block, tiles = (K + 15) / 16;
  const int tile = blockIdx.x % tiles, part = blockIdx.x / tiles;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, r = lane % 16, g = lane / 16;
  const int b = blockIdx.y * 16 + r;  // this lane's sequence
  const int bb = b < a.batch ? b : a.batch - 1;
  const int slot = a.seq_slot[bb], token = a.seq_start[bb];
  const int pos = slot >= 0 ? s.tok_pos[token] : 0, safe = slot >= 0 ? slot : 0;
  const bf16_t* base = s.m.maps + ((size_t)part * 2 * K + min(16 * tile + r, K - 1)) * K + 8 * g;
  f32x4 zr = {0.0f, 0.0f, 0.0f, 0.0f}, zi = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int k = 32 * wave; k < K; k += 32 * 4) {
    bf16x8 u = zero8(), wr = zero8(), wi = zero8();
    if (k + 8 * g < K) {
      float v[8], now[8];
      wr = *(const bf16x8*)(base + k);
      wi = *(const bf16x8*)(base + (size_t)K * K + k);
      unit_input<8>(s, token, safe, pos, part * K + k + 8 * g, v, now);
#pragma unroll
      for (int e = 0; e < 8; ++e) u[e] = (__bf16)v[e];
    }
    zr = mfma(wr, u, zr);
    zi = mfma(wi, u, zi);
  }
  *(f32x4*)&partial[wave][0][lane][0] = zr;
  *(f32x4*)&partial[wave][1][lane][0] = zi;
  __syncthreads();
  if (wave != 0) return;
#pragma unroll
  for (int w = 1; w < 4; ++w) {
    zr += *(const f32x4*)&partial[w][0][lane][0];
    zi += *(const f32x4*)&partial[w][1][lane][0];
  }
  if (b >= a.batch || slot < 0 || 16 * tile + 4 * g >= K) return;
  const int c0 = part * K + 16 * tile + 4 * g;
  float u[4], now[4];
  unit_input<4>(s, token, slot, pos, c0, u, now);
  const f32x4 br = *(const f32x4*)(a.r_bias + c0), bi = *(const f32x4*)(a.i_bias + c0), by = *(const f32x4*)(a.y_bias + c0);
  const f32x4 rate8 = *(const f32x4*)(a.rate + c0) * -8.0f;
  f32x4 S = *(const f32x4*)(a.state + (size_t)slot * a.width + c0);
  const bf16x4 yv = *(const bf16x4*)((const bf16_t*)a.y + (size_t)token * a.y_stride + c0);
  bf16x4 out;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const Decay d = unit_terms(zr[e] + br[e], zi[e] + bi[e], u[e], rate8[e]);
    S[e] = fmaf(d.keep, S[e], d.add);
    out[e] = (__bf16)(S[e] * gelu_tanh_f((float)yv[e] + by[e]));
  }
  *(f32x4*)(a.state + (size_t)slot * a.width + c0) = S;
  *(f32x4*)(s.ring + ((size_t)slot * s.taps + pos % s.taps) * a.width + c0) = (f32x4){now[0], now[1], now[2], now[3]};
  *(bf16x4*)((bf16_t*)a.out + (size_t)token * a.width + c0) = out;
}

}  // namespace

extern "C" int nnis_rg_lru(const float* logits, const float* r_bias, const float* i_bias, const float* rate, const void* u, int u_dtype,
                           int u_stride, const void* y, int y_dtype, int y_stride, const float* y_bias, float* state, const int* seq_slot,
                           const int* seq_start, int batch, int width, int block, void* out, int out_dtype, int piece, int pieces,
                           float* decay, float* ends, void* stream) {
  NNIS_REQUIRE(logits && r_bias && i_bias && rate && u && y && state && seq_slot && seq_start && out, "rg_lru: missing operand");
  NNIS_REQUIRE(nnis_dtype_ok(u_dtype) && nnis_dtype_ok(y_dtype) && nnis_dtype_ok(out_dtype), "rg_lru: unknown dtype");
  NNIS_REQUIRE(width > 0 && block > 0 && width % block == 0 && u_stride >= width && y_stride >= width, "rg_lru: bad sizes (%d channels in blocks of %d)", width, block);
  NNIS_REQUIRE(pieces >= 1 && (pieces == 1 || (piece > 0 && decay && ends)) && (long long)batch * pieces <= 65535, "rg_lru: bad pieces");
  if (batch <= 0) return 0;
  UnitArgs a;
  a.logits = logits; a.r_bias = r_bias; a.i_bias = i_bias; a.rate = rate; a.u = u; a.u_dtype = u_dtype; a.u_stride = u_stride;
  a.y = y; a.y_dtype = y_dtype; a.y_stride = y_stride; a.y_bias = y_bias; a.state = state; a.seq_slot = seq_slot; a.seq_start = seq_start;
  a.batch = batch; a.width = width; a.block = block; a.out = out; a.out_dtype = out_dtype; a.piece = piece; a.pieces = pieces;
  a.decay = decay; a.ends = ends;
  const int threads = width >= 256 ? 256 : 64;
  const dim3 grid((width + threads - 1) / threads, batch * pieces);
  if (pieces > 1) {
    hipLaunchKernelGGL(rg_lru_kernel<1>, grid, dim3(threads), 0, (hipStream_t)stream, a);
    NNIS_LAUNCH_CHECK("rg_lru (first pass)");
  }
  hipLaunchKernelGGL(rg_lru_kernel<2>, grid, dim3(threads), 0, (hipStream_t)stream, a);
  NNIS_LAUNCH_CHECK("rg_lru");
  return 0;
}

static int fill_maps(MapArgs& m, const char* what, const void* maps, const float* r_bias, const float* i_bias, const float* rate, const void* u,
                     int u_stride, const void* y, int y_stride, const float* y_bias, float* state, const int* seq_slot, const int* seq_start,
                     int batch, int width, int block, void* out) {
  NNIS_REQUIRE(maps && r_bias && i_bias && rate && u && y && y_bias && state && seq_slot && seq_start && out, "%s: missing operand", what);
  NNIS_REQUIRE(width > 0 && block > 0 && width % block == 0 && block % 8 == 0 && block <= 512 && u_stride >= width && y_stride >= width && u_stride % 8 == 0 &&
                   y_stride % 8 == 0, "%s: parts of a multiple of 8 channels up to 512 in rows of a multiple of 8, got %d of %d", what, block, width);
  for (const void* p : {maps, (const void*)r_bias, (const void*)i_bias, (const void*)rate, u, y, (const void*)y_bias, (const void*)state, (const void*)out})
    NNIS_REQUIRE((uintptr_t)p % 16 == 0, "%s: operands must be 16-byte aligned", what);
  UnitArgs& a = m.a;
  a.logits = nullptr; a.r_bias = r_bias; a.i_bias = i_bias; a.rate = rate; a.u = u; a.u_dtype = NNIS_BF16; a.u_stride = u_stride;
  a.y = y; a.y_dtype = NNIS_BF16; a.y_stride = y_stride; a.y_bias = y_bias; a.state = state; a.seq_slot = seq_slot; a.seq_start = seq_start;
  a.batch = batch; a.width = width; a.block = block; a.out = out; a.out_dtype = NNIS_BF16; a.piece = 0; a.pieces = 1;
  a.decay = nullptr; a.ends = nullptr;
  m.maps = (const bf16_t*)maps;
  return 0;
}

// maps bfloat16 [blocks, 2 * block, block]; u, y and out bfloat16, y_bias float32
extern "C" int nnis_rg_lru_chunks(const void* maps, const float* r_bias, const float* i_bias, const float* rate, const void* u, int u_stride,
                                  const void* y, int y_stride, const float* y_bias, float* state, const int* seq_slot, const int* seq_start,
                                  int batch, int width, int block, void* out, void* stream) {
  MapArgs m;
  if (fill_maps(m, "rg_lru_chunks", maps, r_bias, i_bias, rate, u, u_stride, y, y_stride, y_bias, state, seq_slot, seq_start, batch, width, block, out)) return 1;
  if (batch <= 0) return 0;
  const int tiles = (block + 15) / 16;
  const long long items = (long long)tiles * (width / block) * batch;
  NNIS_REQUIRE(items <= 0x7ffffff0, "rg_lru_chunks: %d sequences exceed the grid limit", batch);
  const dim3 grid((unsigned)((items + 7) / 8 * 8));
  hipStream_t s = (hipStream_t)stream;
#define NNIS_UNIT(KB_) hipLaunchKernelGGL(rg_lru_chunks_kernel<KB_>, grid, dim3(64 * kWaves), 0, s, m, tiles, (int)items)
  if (block <= 64) NNIS_UNIT(2);
  else if (block <= 128) NNIS_UNIT(4);
  else if (block <= 256) NNIS_UNIT(8);
  else NNIS_UNIT(16);
#undef NNIS_UNIT
  NNIS_LAUNCH_CHECK("rg_lru_chunks");
  return 0;
}

// x: the projection's columns before the convolution and before x_bias; taps_w float32 [taps, width], ring float32 [slots, taps, width]
extern "C" int nnis_rg_lru_step(const void* maps, const float* r_bias, const float* i_bias, const float* rate, const void* x, int x_stride,
                                const void* y, int y_stride, const float* y_bias, const float* x_bias, const float* taps_w, const float* conv_bias,
                                float* ring, float* state, const int* seq_slot, const int* seq_start, const int* tok_pos, int batch, int width,
                                int block, int taps, void* out, void* stream) {
  UnitStepArgs t;
  if (fill_maps(t.m, "rg_lru_step", maps, r_bias, i_bias, rate, x, x_stride, y, y_stride, y_bias, state, seq_slot, seq_start, batch, width, block, out)) return 1;
  NNIS_REQUIRE(x_bias && taps_w && conv_bias && ring && tok_pos && taps > 0, "rg_lru_step: missing operand");
  for (const void* p : {(const void*)x_bias, (const void*)taps_w, (const void*)conv_bias, (const void*)ring})
    NNIS_REQUIRE((uintptr_t)p % 16 == 0, "rg_lru_step: operands must be 16-byte aligned");
  if (batch <= 0) return 0;
  t.x_bias = x_bias; t.taps_w = taps_w; t.conv_bias = conv_bias; t.ring = ring; t.tok_pos = tok_pos; t.taps = taps;
  const dim3 grid((unsigned)((block + 15) / 16 * (width / block)), (unsigned)((batch + 15) / 16));
  hipLaunchKernelGGL(rg_lru_step_kernel, grid, dim3(256), 0, (hipStream_t)stream, t);
  NNIS_LAUNCH_CHECK("rg_lru_step");
  return 0;
}
