// The stream between two sublayers whose norms squash element by element (tanh(alpha v) weight + bias, no statistic over a
// row): the sum of a sublayer's normed output onto the fp32 stream and the next sublayer's normed input in one elementwise
// launch; a pass of a repeated run of layers starts the stream anew from sums of products.
#include "act_types.h"
#include "partial_sums.h"

namespace hymeta {

namespace {

// fp32 activations take the library's tanh.  bf16 ones carry 8 bits: the hardware's exponential, and where its cancellation
// would show the first terms of the series (relative error below 1e-6 on both sides of the seam).
template <typename A>
__device__ __forceinline__ float squash(float v) {
  if (A::kDtype == HYMETA_F32) return tanhf(v);
  const float e = __builtin_amdgcn_exp2f(v * 2.8853900817779268f);          // exp(2 v): inf gives 1, 0 gives -1
  const float far = 1.f - 2.f * __builtin_amdgcn_rcpf(e + 1.f);
  const float s = v * v;
  const float near = v * fmaf(s, fmaf(s, fmaf(s, -17.f / 315.f, 2.f / 15.f), -1.f / 3.f), 1.f);
  return s < 0.0625f ? near : far;
}

template <typename A, int N>
struct Columns;
template <typename A>
struct Columns<A, 4> {
  static __device__ __forceinline__ void ld(const typename A::elem* p, float* v) { A::ld4(p, v); }
  static __device__ __forceinline__ void st(typename A::elem* p, const float* v) { A::st4(p, v); }
};
template <typename A>
struct Columns<A, 1> {
  static __device__ __forceinline__ void ld(const typename A::elem* p, float* v) { v[0] = A::ld(p); }
  static __device__ __forceinline__ void st(typename A::elem* p, const float* v) { A::st(p, v[0]); }
};

// grid = (runs of 256 N columns, strips of R rows): a thread takes N consecutive columns through R rows, the columns'
// constants in registers, the rows' loads in flight together.
// Partials: y is the sum of a K-sliced linear's slabs, added as it is read (N == 4, R == 1).
template <typename A, int N, int R, bool Partials>
__global__ __launch_bounds__(256) void tanh_stream_kernel(hymeta_tanh_stream_args a, hymeta_gemm_partials p) {
  static_assert(!Partials || (N == 4 && R == 1), "slabs are read in fours, a row at a time");
  typedef typename A::elem elem;
  typedef Columns<ActF32, N> F;
  typedef Columns<A, N> E;
  const int c = N * (blockIdx.x * 256 + threadIdx.x);
  const int64_t t0 = static_cast<int64_t>(blockIdx.y) * R;
  if (c >= a.width) return;
  const int rows = min(R, static_cast<int>(a.num_tokens - t0));
  const elem* y = static_cast<const elem*>(a.y);
  elem* h = static_cast<elem*>(a.h_out);
  float v[R][N], yv[R][N];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    if (r >= rows) continue;
    const int64_t t = t0 + r;
    if (a.base) F::ld(a.base + t * a.base_stride_t + c, v[r]);
    else F::ld(a.x + t * a.x_stride_t + c, v[r]);
    if constexpr (Partials) {
      const f32x4 s = partial_row4<false>(p, t, c);
#pragma unroll
      for (int e = 0; e < N; ++e) yv[r][e] = s[e];
    } else if (y) {
      E::ld(y + t * a.y_stride_t + c, yv[r]);
    }
  }
  if (a.base) {
    float add[N];
#pragma unroll
    for (int e = 0; e < N; ++e) add[e] = 0.f;
    if (a.add) F::ld(a.add + c, add);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      if (r >= rows) continue;
      float b2[N];
#pragma unroll
      for (int e = 0; e < N; ++e) b2[e] = 0.f;
      if (a.base2) F::ld(a.base2 + (t0 + r) * a.base_stride_t + c, b2);
#pragma unroll
      for (int e = 0; e < N; ++e) v[r][e] += b2[e] + add[e];
    }
  }
  const bool adds = Partials || y != nullptr;
  if (adds) {
    float w[N], b[N];
    F::ld(a.y_weight + c, w);
    F::ld(a.y_bias + c, b);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      if (r >= rows) continue;
#pragma unroll
      for (int e = 0; e < N; ++e) v[r][e] += fmaf(squash<A>(a.y_alpha * yv[r][e]), w[e], b[e]);
    }
  }
  if (a.base || adds) {
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (r < rows) F::st(a.x + (t0 + r) * a.x_stride_t + c, v[r]);
  }
  if (h) {
    if (a.h_weight) {
      float w[N], b[N];
      F::ld(a.h_weight + c, w);
      F::ld(a.h_bias + c, b);
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < N; ++e) v[r][e] = fmaf(squash<A>(a.h_alpha * v[r][e]), w[e], b[e]);
    }
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (r < rows) E::st(h + (t0 + r) * a.width + c, v[r]);
  }
}

constexpr int kStripRows = 4;

template <typename A, int N>
void launch_tanh_stream(const hymeta_tanh_stream_args& a, hipStream_t st) {
  const int runs = (a.width + 256 * N - 1) / (256 * N);
  // few rows: a row per workgroup, so that there are workgroups enough
  if (a.num_tokens >= 1024) hipLaunchKernelGGL((tanh_stream_kernel<A, N, kStripRows, false>), dim3(runs, (a.num_tokens + kStripRows - 1) / kStripRows), dim3(256), 0, st, a, hymeta_gemm_partials{});
  else hipLaunchKernelGGL((tanh_stream_kernel<A, N, 1, false>), dim3(runs, a.num_tokens), dim3(256), 0, st, a, hymeta_gemm_partials{});
}

inline bool whole_fours(const void* p, int64_t stride, int bytes) { return p == nullptr || (reinterpret_cast<uintptr_t>(p) % (4 * bytes) == 0 && stride % 4 == 0); }
// Everything but y in whole fours of columns.
inline bool stream_in_fours(const hymeta_tanh_stream_args& a, int eb) {
  return a.width % 4 == 0 && whole_fours(a.x, a.x_stride_t, 4) && whole_fours(a.base, a.base_stride_t, 4) && whole_fours(a.base2, a.base_stride_t, 4) &&
         whole_fours(a.add, 0, 4) && whole_fours(a.y_weight, 0, 4) && whole_fours(a.y_bias, 0, 4) && whole_fours(a.h_weight, 0, 4) &&
         whole_fours(a.h_bias, 0, 4) && whole_fours(a.h_out, 0, eb);
}

}  // namespace

}  // namespace hymeta

using namespace hymeta;

extern "C" int hymeta_tanh_stream(const hymeta_tanh_stream_args* args, hymeta_stream_t stream) {
  if (!args_ok(args)) return HYMETA_ERR_INVALID_ARG;
  const hymeta_tanh_stream_args& a = *args;
  if (a.num_tokens < 0 || a.width <= 0) return HYMETA_ERR_INVALID_ARG;
  if (!act_dtype_ok(a.act_dtype)) return HYMETA_ERR_UNSUPPORTED;
  if (a.num_tokens == 0) return HYMETA_OK;
  if (!a.x || a.x_stride_t < a.width || (!a.y && !a.base && !a.h_out)) return HYMETA_ERR_INVALID_ARG;
  if (a.y && (!a.y_weight || !a.y_bias || a.y_stride_t < a.width)) return HYMETA_ERR_INVALID_ARG;
  if (a.base ? a.base_stride_t < a.width : (a.base2 != nullptr || a.add != nullptr)) return HYMETA_ERR_INVALID_ARG;
  if (a.h_weight && !a.h_bias) return HYMETA_ERR_INVALID_ARG;
  if ((a.num_tokens + kStripRows - 1) / kStripRows > 65535) return HYMETA_ERR_UNSUPPORTED;
  hipStream_t st = begin_launches(stream);
  const int eb = a.act_dtype == HYMETA_BF16 ? 2 : 4;
  const bool vec = stream_in_fours(a, eb) && whole_fours(a.y, a.y_stride_t, eb);
  if (a.act_dtype == HYMETA_BF16) {
    if (vec) launch_tanh_stream<ActBf16, 4>(a, st);
    else launch_tanh_stream<ActBf16, 1>(a, st);
  } else {
    if (vec) launch_tanh_stream<ActF32, 4>(a, st);
    else launch_tanh_stream<ActF32, 1>(a, st);
  }
  return launch_status();
}

extern "C" int hymeta_tanh_stream_partials(const hymeta_tanh_stream_args* args, const hymeta_gemm_partials* partials, hymeta_stream_t stream) {
  if (!args_ok(args) || !args_ok(partials)) return HYMETA_ERR_INVALID_ARG;
  const hymeta_tanh_stream_args& a = *args;
  const hymeta_gemm_partials& p = *partials;
  if (a.num_tokens < 0 || a.width <= 0 || p.splits <= 0 || p.is_int32 || !p.slabs || p.M != a.num_tokens || p.N != a.width) return HYMETA_ERR_INVALID_ARG;
  if (a.act_dtype != HYMETA_BF16) return HYMETA_ERR_UNSUPPORTED;
  if (a.num_tokens == 0) return HYMETA_OK;
  if (!a.x || a.x_stride_t < a.width || !a.y_weight || !a.y_bias || a.base || a.base2 || a.add || (a.h_weight && !a.h_bias)) return HYMETA_ERR_INVALID_ARG;
  if (!stream_in_fours(a, 2) || reinterpret_cast<uintptr_t>(p.slabs) % 16 != 0 || !whole_fours(p.bias, 0, 2) || a.num_tokens > 65535) return HYMETA_ERR_UNSUPPORTED;
  hipStream_t st = begin_launches(stream);
  hipLaunchKernelGGL((tanh_stream_kernel<ActBf16, 4, 1, true>), dim3((a.width + 1023) / 1024, a.num_tokens), dim3(256), 0, st, a, p);
  return launch_status();
}
