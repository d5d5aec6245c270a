// Shared device helpers for the gfx950 kernels: storage types, conversions, wave64 reductions,
// and the error channel of the C entry points.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace kvcm {

constexpr int kWave = 64;

// Storage types.  bf16 is kept as raw bits so that loads can be vectorised freely.
struct bf16_t { uint16_t bits; };

enum DType : int { kF32 = 0, kBF16 = 1 };

__device__ __forceinline__ float bf16_bits_to_float(uint32_t b) { return __uint_as_float(b << 16); }
// Round to nearest, ties to even; a NaN stays a quiet NaN.  gfx950 converts in one instruction
// (v_cvt_pk_bf16_f32); written out in integer operations it costs six and a branch, which epilogues
// that round a dozen values per lane pay in microseconds.
__device__ __forceinline__ uint16_t float_to_bf16_bits(float f) {
  return __builtin_bit_cast(uint16_t, static_cast<__bf16>(f));
}

template <class T> __device__ __forceinline__ float load_f(const T* p);
template <> __device__ __forceinline__ float load_f<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float load_f<bf16_t>(const bf16_t* p) { return bf16_bits_to_float(p->bits); }

template <class T> __device__ __forceinline__ void store_f(T* p, float v);
template <> __device__ __forceinline__ void store_f<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void store_f<bf16_t>(bf16_t* p, float v) { p->bits = float_to_bf16_bits(v); }

// Value after one trip through the storage type (identity for float).
template <class T> __device__ __forceinline__ float round_to(float v);
template <> __device__ __forceinline__ float round_to<float>(float v) { return v; }
template <> __device__ __forceinline__ float round_to<bf16_t>(float v) { return bf16_bits_to_float(float_to_bf16_bits(v)); }

// silu(x) = x / (1 + exp(-x)) for a result stored as T.  A bfloat16 result keeps 8 bits of it: the
// hardware's exp2 and reciprocal (about 1 ulp of float each) take a tenth of the instructions of the
// exact functions, which in a product's epilogue is microseconds (a 64-lane wave spends 4 cycles
// per instruction).  A float result takes the exact functions.  One definition for every kernel
// that applies it, so that all of them give the same bits.
template <class T> __device__ __forceinline__ float silu(float x);
template <> __device__ __forceinline__ float silu<float>(float x) { return x / (1.0f + expf(-x)); }
template <> __device__ __forceinline__ float silu<bf16_t>(float x) {
  return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.44269504088896341f * x));
}

// Activations of feed-forwards by number, in 32-bit: 0 silu, 1 relu, 2 gelu by tanh (0.5 z (1 + tanh(sqrt(2/pi) (z +
// 0.044715 z^3)))), 3 gelu by the error function (z times the normal distribution's function of z).
__device__ __forceinline__ float ff_activation(int act, float z) {
  if (act == 1) return fmaxf(z, 0.f);
  if (act == 2) return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  if (act == 3) return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f));
  return z / (1.0f + expf(-z));
}

// The exact gelu for a result stored as T.  For a bfloat16 result the error function is the five-term approximation of
// Abramowitz and Stegun's handbook (formula 7.1.26, absolute error up to 1.5e-7) in its complementary form, with the hardware's
// exp2 and reciprocal: erfc(x) = (a1 t + .. + a5 t^5) exp(-x^2), t = 1 / (1 + p x), x >= 0.
template <class T> __device__ __forceinline__ float gelu_exact(float z);
template <> __device__ __forceinline__ float gelu_exact<float>(float z) { return ff_activation(3, z); }
template <> __device__ __forceinline__ float gelu_exact<bf16_t>(float z) {
  const float x = fabsf(z) * 0.70710678118654752f;
  const float t = __builtin_amdgcn_rcpf(fmaf(0.3275911f, x, 1.0f));
  const float poly = t * fmaf(t, fmaf(t, fmaf(t, fmaf(t, 1.061405429f, -1.453152027f), 1.421413741f), -0.284496736f), 0.254829592f);
  const float half_erfc = 0.5f * poly * __builtin_amdgcn_exp2f(-1.44269504088896341f * x * x);      // the distribution's tail beyond |z|
  return z * (z < 0.f ? half_erfc : 1.0f - half_erfc);
}

// A gate with limits: g = min(gate, limit), u = up held within [-limit, limit], g / (1 + exp(-1.702 g)) * (u + 1).
constexpr float kClampedGateSlope = 1.702f;
template <class T> __device__ __forceinline__ float clamped_gate(float gate, float up, float limit) {
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return silu<T>(kClampedGateSlope * g) * (1.0f / kClampedGateSlope) * (u + 1.0f);
}

// (a, b) rotated by the angle whose cosine and sine are given.  One explicit sequence of
// operations, shared by every kernel that rotates, so that all of them give the same bits.
__device__ __forceinline__ void rotate_pair(float& a, float& b, float cs, float sn) {
  const float ra = __fmaf_rn(a, cs, -__fmul_rn(b, sn));
  const float rb = __fmaf_rn(b, cs, __fmul_rn(a, sn));
  a = ra;
  b = rb;
}

// A 16-byte piece of 8 bfloat16 with only its first n (0..8) kept, the others zero.  Value pieces that
// reach past a context's end hold whatever the page's previous owner left there; their probabilities
// are zero, but zero times a stale Inf or NaN would not be: such pieces are cut before they are multiplied.
__device__ __forceinline__ uint4 keep_first_bf16(uint4 v, int n) {
  auto word = [n](int j) -> uint32_t { return n >= 2 * j + 2 ? 0xFFFFFFFFu : (n == 2 * j + 1 ? 0x0000FFFFu : 0u); };
  return uint4{v.x & word(0), v.y & word(1), v.z & word(2), v.w & word(3)};
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = kWave / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, kWave);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = kWave / 2; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, kWave));
  return v;
}

// Sum over aligned groups of G lanes (a power of two); every lane of a group gets the result.  Up to 16 lanes the
// partners come by data-parallel-primitive moves inside a row of 16 (a few cycles each: lane ^ 1, lane ^ 2, then the
// mirrored half and the mirrored row, whose lanes hold the other half's sum already); beyond that by shuffles.
template <int CTRL>
__device__ __forceinline__ float dpp_take(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}
template <int G>
__device__ __forceinline__ float group_sum(float v) {
  if constexpr (G >= 2) v += dpp_take<0xB1>(v);       // quad_perm [1, 0, 3, 2]
  if constexpr (G >= 4) v += dpp_take<0x4E>(v);       // quad_perm [2, 3, 0, 1]
  if constexpr (G >= 8) v += dpp_take<0x141>(v);      // row_half_mirror
  if constexpr (G >= 16) v += dpp_take<0x140>(v);     // row_mirror
  if constexpr (G >= 32) v += __shfl_xor(v, 16, kWave);
  if constexpr (G >= 64) v += __shfl_xor(v, 32, kWave);
  return v;
}

template <int G>
__device__ __forceinline__ float group_max(float v) {      // as group_sum, the largest instead of the sum
  if constexpr (G >= 2) v = fmaxf(v, dpp_take<0xB1>(v));
  if constexpr (G >= 4) v = fmaxf(v, dpp_take<0x4E>(v));
  if constexpr (G >= 8) v = fmaxf(v, dpp_take<0x141>(v));
  if constexpr (G >= 16) v = fmaxf(v, dpp_take<0x140>(v));
  if constexpr (G >= 32) v = fmaxf(v, __shfl_xor(v, 16, kWave));
  if constexpr (G >= 64) v = fmaxf(v, __shfl_xor(v, 32, kWave));
  return v;
}

// Sum over a block of THREADS threads (a multiple of 64); every thread gets the result.  The
// order of additions depends on THREADS only.
template <int THREADS>
__device__ __forceinline__ float block_sum(float v, float* scratch /* THREADS/64 + 1 floats */) {
  v = wave_sum(v);
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  if (threadIdx.x == 0) {
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < THREADS / kWave; ++w) s += scratch[w];
    scratch[THREADS / kWave] = s;
  }
  __syncthreads();
  const float r = scratch[THREADS / kWave];
  __syncthreads();
  return r;
}

// ---- host side ------------------------------------------------------------------------------
void set_error(const char* fmt, ...);
int launch_status(const char* what);

}  // namespace kvcm

#define KVCM_REQUIRE(cond, ...)          \
  do {                                   \
    if (!(cond)) {                       \
      kvcm::set_error(__VA_ARGS__);      \
      return -1;                         \
    }                                    \
  } while (0)
