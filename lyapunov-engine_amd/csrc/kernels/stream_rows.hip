// The residual stream between two branches, and logits after their product:
// work that needs no sum over a row.  All arithmetic is 32-bit; only loads and
// stores see the storage type.
//
//   * stream_map: v = base + delta (delta in the activations' type, float, or float partial sums
//     that are added up in their order), v to h where h is given, and the following branch's input
//     map(v) (stream_map.h) to out.  base may be h itself or another tensor: a stream that starts
//     afresh.  With `rows` only those rows are mapped and h is left alone.
//   * logit_cap: z <- cap * tanh(scale * z / cap), or scale * z without a cap, in place.
#include <algorithm>

#include "stream_map.h"

namespace lyp {

constexpr int kMapThreads = 256;

// V neighbouring features a thread; blockIdx.y walks the row in pieces of kMapThreads * V.
template <typename TD, typename T, int V>
__global__ __launch_bounds__(kMapThreads) void stream_map_kernel(float* h, const float* base,
                                                                 const TD* __restrict__ delta, int n_parts,
                                                                 size_t part_stride, StreamMap map, T* __restrict__ out,
                                                                 const int32_t* __restrict__ rows, int H) {
  typedef float VecF __attribute__((ext_vector_type(V)));
  typedef TD VecD __attribute__((ext_vector_type(V)));
  typedef T VecT __attribute__((ext_vector_type(V)));
  const int c = (blockIdx.y * kMapThreads + threadIdx.x) * V;
  if (c >= H) return;
  const int r = blockIdx.x;
  const size_t src = (rows != nullptr ? static_cast<size_t>(rows[r]) : static_cast<size_t>(r)) * H + c;
  VecF v = *reinterpret_cast<const VecF*>(base + src);
  VecF w, b;
  if (map.kind == kMapTanh && out != nullptr) {
    w = *reinterpret_cast<const VecF*>(map.w + c);
    b = *reinterpret_cast<const VecF*>(map.b + c);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) w[i] = b[i] = 0.f;
  }
  if (delta != nullptr) {
    // the partial sums first, in their order, then the stream
    VecF d;
#pragma unroll
    for (int i = 0; i < V; ++i) d[i] = 0.f;
    for (int p = 0; p < n_parts; ++p) {
      const VecD x = *reinterpret_cast<const VecD*>(delta + p * part_stride + src);
#pragma unroll
      for (int i = 0; i < V; ++i) d[i] += to_f32(x[i]);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] += d[i];
  }
  if (h != nullptr) *reinterpret_cast<VecF*>(h + src) = v;
  if (out == nullptr) return;
  VecT o;
#pragma unroll
  for (int i = 0; i < V; ++i) o[i] = from_f32<T>(map_feature(map.kind, map.alpha, v[i], w[i], b[i]));
  *reinterpret_cast<VecT*>(out + static_cast<size_t>(r) * H + c) = o;
}

__global__ void logit_cap_kernel(float* __restrict__ z, size_t n, float scale, float cap) {
  const size_t stride = static_cast<size_t>(gridDim.x) * blockDim.x;
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < n; i += stride)
    z[i] = shaped_logit(z[i], scale, cap);
}

}  // namespace lyp

using namespace lyp;

extern "C" {

// base float [T, H]; delta [T, H] of delta_dtype or n_parts partial sums part_stride apart, or null;
// h float [T, H] or null (the sum is not kept; with rows it must be null); out [n_rows, H] of
// out_dtype or null.  kind 0: out = v; kind 1: out = tanh(alpha v) w + b with w, b float [H].
int lyp_stream_map(float* h, const float* base, const void* delta, int delta_dtype, int n_parts, long long part_stride,
                   int kind, float alpha, const float* w, const float* b, void* out, int out_dtype, const int32_t* rows,
                   int n_rows, int H, hipStream_t stream) {
  const StreamMap map{kind, alpha, w, b};
  LYP_REQUIRE(n_rows >= 0 && H > 0 && base != nullptr && n_parts >= 0 && part_stride >= 0, "stream_map: bad sizes");
  LYP_REQUIRE(out == nullptr || stream_map_ok(map), "stream_map: kind %d needs its vectors", kind);
  LYP_REQUIRE(h == nullptr || rows == nullptr, "stream_map: picked rows leave the stream alone");
  LYP_REQUIRE(h != nullptr || out != nullptr, "stream_map: nothing to write");
  if (n_rows == 0) return 0;
  auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = H % 4 == 0 && part_stride % 4 == 0 && aligned(h) && aligned(base) && aligned(delta) && aligned(w) &&
                   aligned(b) && aligned(out);
  const int per = vec ? 4 : 1;
  const dim3 grid(n_rows, (H + kMapThreads * per - 1) / (kMapThreads * per));
#define LYP_MAP(TD, T)                                                                                              \
  do {                                                                                                              \
    if (vec)                                                                                                        \
      stream_map_kernel<TD, T, 4><<<grid, kMapThreads, 0, stream>>>(h, base, static_cast<const TD*>(delta), n_parts,  \
                                                                    static_cast<size_t>(part_stride), map,          \
                                                                    static_cast<T*>(out), rows, H);                 \
    else                                                                                                            \
      stream_map_kernel<TD, T, 1><<<grid, kMapThreads, 0, stream>>>(h, base, static_cast<const TD*>(delta), n_parts,  \
                                                                    static_cast<size_t>(part_stride), map,          \
                                                                    static_cast<T*>(out), rows, H);                 \
  } while (0)
  if (delta_dtype == kF32 && out_dtype == kF32) LYP_MAP(float, float);
  else if (delta_dtype == kF32 && out_dtype == kBF16) LYP_MAP(float, bf16_t);
  else if (delta_dtype == kBF16 && out_dtype == kF32) LYP_MAP(bf16_t, float);
  else if (delta_dtype == kBF16 && out_dtype == kBF16) LYP_MAP(bf16_t, bf16_t);
  else LYP_REQUIRE(false, "stream_map: unknown dtypes %d, %d", delta_dtype, out_dtype);
#undef LYP_MAP
  LYP_LAUNCH_CHECK("stream_map");
  return 0;
}

// z float [n], in place; cap 0: no cap.
int lyp_logit_cap(float* z, long long n, float scale, float cap, hipStream_t stream) {
  LYP_REQUIRE(n >= 0 && cap >= 0.f, "logit_cap: n=%lld cap=%f", n, static_cast<double>(cap));
  if (n == 0) return 0;
  const int blocks = static_cast<int>(std::min<long long>((n + 255) / 256, 16384));
  logit_cap_kernel<<<blocks, 256, 0, stream>>>(z, static_cast<size_t>(n), scale, cap);
  LYP_LAUNCH_CHECK("logit_cap");
  return 0;
}

}  // extern "C"
