// The stream of layers whose sublayers all read one normed copy of it, x <- x + sum of their outputs:
//
//   stream_terms   x <- x + (fa * a + fb * b + fc * c + bias), up to three terms with a factor each and a constant row, and
//                  then, at the start of a stretch that runs again, x <- x + x0 (the embedding's output); and in the same
//                  launch the RMS norm that the next sublayers read, out = x / sqrt(mean(x^2) + eps) * w.  A term may be
//                  the un-added slices of a product that was split along K: they are added here, in their order.  With a
//                  row gather (the model's last norm, on the rows whose logits are wanted) nothing is written back.
//   group_norm_gate  a gate before a norm: v = y * silu(z), then groups of consecutive columns of v are divided by their
//                  root mean square and weighted; or (after) the norm first, v = y, and then the factor sigmoid(z).
//
// All arithmetic is 32-bit; a row's result is one fixed sequence of operations on that row alone.
#include "common.h"
#include "kvcm_hip.h"

namespace kvcm {

constexpr int kTermThreads = 256;

struct Terms {
  const float* p[3];
  int splits[3];
  float factor[3];
  size_t split_stride;
  const float* bias;
  const float* again;
};

// sum over the workgroup with one barrier: every thread adds the waves' sums itself, in wave order
__device__ __forceinline__ float terms_block_sum(float v, float* scratch /* kTermThreads / 64 floats of this sum's own */) {
  v = wave_sum(v);
  if (threadIdx.x % kWave == 0) scratch[threadIdx.x / kWave] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int w = 0; w < kTermThreads / kWave; ++w) s += scratch[w];
  return s;
}

// any row length: a value is formed as often as it is needed
template <class TO>
__global__ void __launch_bounds__(kTermThreads)
    stream_terms_kernel(float* __restrict__ x, Terms t, const int* __restrict__ rows, const float* __restrict__ w,
                        TO* __restrict__ out, int H, float eps, int write_back) {
  __shared__ float scratch[kTermThreads / kWave];
  const int r = blockIdx.x;
  const size_t src = size_t(rows ? rows[r] : r) * H;
  auto value = [&](int i) {
    float sum = 0.f;
    for (int k = 0; k < 3; ++k) {
      if (!t.p[k]) continue;
      float v = t.p[k][src + i];
      for (int sl = 1; sl < t.splits[k]; ++sl) v += t.p[k][size_t(sl) * t.split_stride + src + i];
      sum = fmaf(t.factor[k], v, sum);
    }
    if (t.bias) sum += t.bias[i];
    float v = x[src + i] + sum;
    if (t.again) v += t.again[src + i];
    return v;
  };
  float ss = 0.f;
  if (out) {
    for (int i = threadIdx.x; i < H; i += kTermThreads) {
      const float v = value(i);
      ss = fmaf(v, v, ss);
    }
    ss = terms_block_sum(ss, scratch);
  }
  const float inv = 1.0f / sqrtf(ss / float(H) + eps);
  for (int i = threadIdx.x; i < H; i += kTermThreads) {      // an element is read and written by one thread only
    const float v = value(i);
    if (write_back) x[src + i] = v;
    if (out) store_f(out + size_t(r) * H + i, v * inv * w[i]);
  }
}

// rows of a multiple of four values, at most 1024 * G of them: read once, 16 bytes a load, kept in registers
template <class TO, int G>
__global__ void __launch_bounds__(kTermThreads)
    stream_terms_rows_kernel(float* __restrict__ x, Terms t, const int* __restrict__ rows, const float* __restrict__ w,
                             TO* __restrict__ out, int H, float eps, int write_back) {
  __shared__ float scratch[kTermThreads / kWave];
  const int r = blockIdx.x;
  const size_t src = size_t(rows ? rows[r] : r) * H;
  float v[G][4];
  bool in[G];
#pragma unroll
  for (int g = 0; g < G; ++g) {
    const int i = (g * kTermThreads + threadIdx.x) * 4;
    in[g] = i < H;
    const size_t at = src + (in[g] ? i : 0);
    float4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 3; ++k) {
      if (!t.p[k]) continue;
      const float* p = t.p[k] + at;
      float4 y = *reinterpret_cast<const float4*>(p);
#pragma unroll 4
      for (int sl = 1; sl < t.splits[k]; ++sl) {
        const float4 a = *reinterpret_cast<const float4*>(p + size_t(sl) * t.split_stride);
        y.x += a.x; y.y += a.y; y.z += a.z; y.w += a.w;
      }
      const float f = t.factor[k];
      sum.x = fmaf(f, y.x, sum.x); sum.y = fmaf(f, y.y, sum.y); sum.z = fmaf(f, y.z, sum.z); sum.w = fmaf(f, y.w, sum.w);
    }
    if (t.bias) {
      const float4 b = *reinterpret_cast<const float4*>(t.bias + (in[g] ? i : 0));
      sum.x += b.x; sum.y += b.y; sum.z += b.z; sum.w += b.w;
    }
    const float4 xv = *reinterpret_cast<const float4*>(x + at);
    v[g][0] = xv.x + sum.x; v[g][1] = xv.y + sum.y; v[g][2] = xv.z + sum.z; v[g][3] = xv.w + sum.w;
    if (t.again) {
      const float4 a = *reinterpret_cast<const float4*>(t.again + at);
      v[g][0] += a.x; v[g][1] += a.y; v[g][2] += a.z; v[g][3] += a.w;
    }
    if (write_back && in[g]) *reinterpret_cast<float4*>(x + at) = float4{v[g][0], v[g][1], v[g][2], v[g][3]};
  }
  if (!out) return;
  float ss = 0.f;
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (in[g]) ss = fmaf(v[g][e], v[g][e], ss);
  const float inv = 1.0f / sqrtf(terms_block_sum(ss, scratch) / float(H) + eps);
#pragma unroll
  for (int g = 0; g < G; ++g) {
    if (!in[g]) continue;
    const int i = (g * kTermThreads + threadIdx.x) * 4;
    const float4 ww = *reinterpret_cast<const float4*>(w + i);
    TO* o = out + size_t(r) * H + i;
    store_f(o, v[g][0] * inv * ww.x); store_f(o + 1, v[g][1] * inv * ww.y);
    store_f(o + 2, v[g][2] * inv * ww.z); store_f(o + 3, v[g][3] * inv * ww.w);
  }
}

// one workgroup per (row, group); groups of up to 256 HELD values are read once, all loads on their way together, and kept in
// registers
template <class TO, int HELD>
__global__ void __launch_bounds__(kTermThreads)
    group_norm_gate_kernel(const float* __restrict__ y, int ldy, const float* __restrict__ z, int ldz, const float* __restrict__ w,
                           TO* __restrict__ out, int ldo, int size, float eps, int after) {
  __shared__ float scratch[kTermThreads / kWave];
  const int row = blockIdx.x, c0 = blockIdx.y * size;
  const float* yr = y + size_t(row) * ldy + c0;
  const float* zr = z + size_t(row) * ldz + c0;
  TO* o = out + size_t(row) * ldo + c0;
  auto value = [&](int i) {
    if (after) return yr[i];
    const float g = zr[i];
    return yr[i] * (g / (1.0f + expf(-g)));
  };
  if (size <= HELD * kTermThreads) {
    float v[HELD], z4[HELD], ss = 0.f;
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
      const int i = threadIdx.x + j * kTermThreads, ic = i < size ? i : 0;
      v[j] = yr[ic];
      z4[j] = zr[ic];
    }
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
      const int i = threadIdx.x + j * kTermThreads;
      const float sg = 1.0f / (1.0f + expf(-z4[j]));
      v[j] = i < size ? (after ? v[j] : v[j] * (z4[j] * sg)) : 0.f;
      z4[j] = after ? sg : 1.f;
      ss = fmaf(v[j], v[j], ss);
    }
    const float inv = 1.0f / sqrtf(terms_block_sum(ss, scratch) / float(size) + eps);
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
      const int i = threadIdx.x + j * kTermThreads;
      if (i < size) store_f(o + i, v[j] * inv * w[c0 + i] * z4[j]);
    }
    return;
  }
  float ss = 0.f;
  for (int i = threadIdx.x; i < size; i += kTermThreads) {
    const float v = value(i);
    ss = fmaf(v, v, ss);
  }
  const float inv = 1.0f / sqrtf(terms_block_sum(ss, scratch) / float(size) + eps);
  for (int i = threadIdx.x; i < size; i += kTermThreads)
    store_f(o + i, value(i) * inv * w[c0 + i] * (after ? 1.0f / (1.0f + expf(-zr[i])) : 1.f));
}

}  // namespace kvcm

using namespace kvcm;

extern "C" {

// x [T, H] 32-bit.  a, b, c: terms [T, H] or their un-added slices [splits][T][H], split_stride floats apart (null: absent);
// bias [H] or null; again [T, H] or null; rows: source rows of the R outputs (null: row r, and x is updated in place where
// anything is added); out [R, H] in out_dtype with its weight w [H], or null.
int kvcm_stream_terms(float* x, const float* a, int a_splits, float a_factor, const float* b, int b_splits, float b_factor,
                      const float* c, int c_splits, float c_factor, long long split_stride, const float* bias, const float* again,
                      const int* rows, const float* w, void* out, int out_dtype, int R, int H, float eps, hipStream_t s) {
  if (R == 0) return 0;
  KVCM_REQUIRE(R > 0 && H > 0 && x, "stream_terms: bad sizes R=%d H=%d", R, H);
  KVCM_REQUIRE(a_splits >= 1 && b_splits >= 1 && c_splits >= 1 && split_stride >= 0, "stream_terms: a term has at least one slice");
  KVCM_REQUIRE(!out || w, "stream_terms: a normed output needs its weight");
  KVCM_REQUIRE(out || !rows, "stream_terms: gathered rows need an output");
  KVCM_REQUIRE(!out || out_dtype == kF32 || out_dtype == kBF16, "stream_terms: unknown output dtype %d", out_dtype);
  const Terms t = {{a, b, c}, {a_splits, b_splits, c_splits}, {a_factor, b_factor, c_factor}, static_cast<size_t>(split_stride), bias, again};
  const int write_back = !rows && (a || b || c || bias || again) ? 1 : 0;
  KVCM_REQUIRE(out || write_back, "stream_terms: nothing to do");
  const bool f32 = !out || out_dtype == kF32;
  auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (H % 4 == 0 && H <= 8192 && split_stride % 4 == 0 && aligned(x) && aligned(a) && aligned(b) && aligned(c) && aligned(bias) &&
      aligned(again) && aligned(w)) {
#define KVCM_TERM_ROWS(TO, G) \
  stream_terms_rows_kernel<TO, G><<<R, kTermThreads, 0, s>>>(x, t, rows, w, static_cast<TO*>(out), H, eps, write_back)
    if (H <= 2048) { if (f32) KVCM_TERM_ROWS(float, 2); else KVCM_TERM_ROWS(bf16_t, 2); }
    else if (H <= 4096) { if (f32) KVCM_TERM_ROWS(float, 4); else KVCM_TERM_ROWS(bf16_t, 4); }
    else { if (f32) KVCM_TERM_ROWS(float, 8); else KVCM_TERM_ROWS(bf16_t, 8); }
#undef KVCM_TERM_ROWS
    return launch_status("stream_terms");
  }
  if (f32) stream_terms_kernel<float><<<R, kTermThreads, 0, s>>>(x, t, rows, w, static_cast<float*>(out), H, eps, write_back);
  else stream_terms_kernel<bf16_t><<<R, kTermThreads, 0, s>>>(x, t, rows, w, static_cast<bf16_t*>(out), H, eps, write_back);
  return launch_status("stream_terms");
}

// y, z [T, >= groups * size] 32-bit rows; w [groups * size]; out [T, >= groups * size] in out_dtype
int kvcm_group_norm_gate(const float* y, int ldy, const float* z, int ldz, const float* w, void* out, int out_dtype, int ldo, int T,
                         int groups, int size, float eps, int after, hipStream_t s) {
  if (T == 0) return 0;
  KVCM_REQUIRE(T > 0 && groups > 0 && size > 0 && y && z && w && out, "group_norm_gate: bad sizes T=%d groups=%d size=%d", T, groups, size);
  KVCM_REQUIRE(groups <= 65535 && ldy >= groups * size && ldz >= groups * size && ldo >= groups * size, "group_norm_gate: row strides too small");
  const dim3 grid(T, groups);
#define KVCM_GROUP_NORM(TO)                                                                                                        \
  {                                                                                                                                \
    TO* oo = static_cast<TO*>(out);                                                                                                \
    if (size <= 1024) group_norm_gate_kernel<TO, 4><<<grid, kTermThreads, 0, s>>>(y, ldy, z, ldz, w, oo, ldo, size, eps, after);    \
    else if (size <= 2048) group_norm_gate_kernel<TO, 8><<<grid, kTermThreads, 0, s>>>(y, ldy, z, ldz, w, oo, ldo, size, eps, after); \
    else group_norm_gate_kernel<TO, 16><<<grid, kTermThreads, 0, s>>>(y, ldy, z, ldz, w, oo, ldo, size, eps, after);                \
  }
  if (out_dtype == kF32) KVCM_GROUP_NORM(float)
  else if (out_dtype == kBF16) KVCM_GROUP_NORM(bf16_t)
  else KVCM_REQUIRE(false, "group_norm_gate: unknown output dtype %d", out_dtype);
#undef KVCM_GROUP_NORM
  return launch_status("group_norm_gate");
}

}  // extern "C"
