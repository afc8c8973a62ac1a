// A residual of several streams (hyper-connections): instead of one row x a token has S rows x_1 .. x_S. A sublayer
// reads one mixture of them, u = sum_s in[s] x_s, and its result y goes back to all of them while they are mixed with
// each other, x_t <- sum_s mix[s][t] x_s + out[t] y. One kernel stands between two sublayers:
//
//   x    <- the streams after the sublayer before (its result as partial sums, its mix and out; or no such sublayer)
//   u     = sum_s in[s] x_s                  (in = null: the plain sum)
//   rows  = (u - mean) / sqrt(mean((u - mean)^2) + eps) * gain (+ shift), or without the mean (an RMS norm)
//
// so that the streams are read and written once per sublayer. `src` may be one row a token (src_streams = 1: all
// streams are equal, as they are behind the embedding); with `picked` only the listed rows are normed and nothing is
// written back. Everything float32; a row's sums are block sums of per-thread sums.
#include "pyre_api.h"
#include "pyre_common.h"
#include "pyre_vec4.h"

using namespace pyre;

namespace {

constexpr int kMaxStreams = 8;

// One row's elements are dealt to THREADS x ITEMS float4 (VEC) or single floats; an element's streams (up to S of
// them) are in registers together.
template <typename TD, typename TO, int S, int THREADS, int ITEMS, bool VEC>
__global__ __launch_bounds__(THREADS) void stream_norm_kernel(
    const float* __restrict__ src, int src_streams, float* __restrict__ dst, int streams, const TD* __restrict__ y, int n_partials,
    size_t partial_stride, const float* __restrict__ mix, const float* __restrict__ out_w, const float* __restrict__ in_w,
    const float* __restrict__ gain, const float* __restrict__ shift, int center, float eps, TO* __restrict__ out,
    const int* __restrict__ picked, int hidden) {
  constexpr int W = VEC ? 4 : 1;
  __shared__ float scratch[16];
  const int r_out = blockIdx.x, r_in = picked ? picked[r_out] : r_out, tid = threadIdx.x;
  const size_t row = static_cast<size_t>(r_in) * hidden;
  const float inv_n = 1.f / static_cast<float>(hidden);
  float u[ITEMS][W];
  float mixed[S][S], back[S], into[S];
#pragma unroll
  for (int t = 0; t < S; ++t) {
    into[t] = t < streams ? (in_w ? in_w[t] : 1.f) : 0.f;
    back[t] = y && t < streams ? out_w[t] : 0.f;
#pragma unroll
    for (int s = 0; s < S; ++s) mixed[s][t] = y && s < streams && t < streams ? mix[s * streams + t] : 0.f;
  }
#pragma unroll
  for (int k = 0; k < ITEMS; ++k) {
    const int i = W * (tid + k * THREADS);
#pragma unroll
    for (int e = 0; e < W; ++e) u[k][e] = 0.f;
    if (i >= hidden) continue;
    float x[S][W], d[W];
#pragma unroll
    for (int s = 0; s < S; ++s) {
#pragma unroll
      for (int e = 0; e < W; ++e) x[s][e] = 0.f;
      if (s >= streams) continue;
      const float* p = src + (src_streams == 1 ? row : (static_cast<size_t>(r_in) * streams + s) * hidden) + i;
      if constexpr (VEC) {
        const float4 v = Vec4<float>::load(p);
        x[s][0] = v.x, x[s][1] = v.y, x[s][2] = v.z, x[s][3] = v.w;
      } else {
        x[s][0] = *p;
      }
    }
    if (y) {
      if constexpr (VEC) {
        const float4 v = sum_partials4(y + row + i, partial_stride, n_partials);
        d[0] = v.x, d[1] = v.y, d[2] = v.z, d[3] = v.w;
      } else {
        d[0] = 0.f;
        for (int p = 0; p < n_partials; ++p) d[0] += to_float(y[p * partial_stride + row + i]);
      }
      float z[S][W];
#pragma unroll
      for (int t = 0; t < S; ++t)
#pragma unroll
        for (int e = 0; e < W; ++e) {
          float v = back[t] * d[e];
#pragma unroll
          for (int s = 0; s < S; ++s) v = fmaf(mixed[s][t], x[s][e], v);
          z[t][e] = v;
        }
#pragma unroll
      for (int t = 0; t < S; ++t) {
#pragma unroll
        for (int e = 0; e < W; ++e) x[t][e] = z[t][e];
        if (dst && t < streams) {
          float* p = dst + (static_cast<size_t>(r_in) * streams + t) * hidden + i;
          if constexpr (VEC) Vec4<float>::store(p, float4{x[t][0], x[t][1], x[t][2], x[t][3]});
          else *p = x[t][0];
        }
      }
    }
#pragma unroll
    for (int s = 0; s < S; ++s)
#pragma unroll
      for (int e = 0; e < W; ++e) u[k][e] = fmaf(into[s], x[s][e], u[k][e]);
  }
  float mean = 0.f;
  if (center) {
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < ITEMS; ++k)
#pragma unroll
      for (int e = 0; e < W; ++e) sum += u[k][e];  // elements behind the row's end are zero
    mean = block_sum(sum, scratch) * inv_n;
  }
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < ITEMS; ++k)
    if (W * (tid + k * THREADS) < hidden)
#pragma unroll
      for (int e = 0; e < W; ++e) ss += (u[k][e] - mean) * (u[k][e] - mean);
  const float inv = 1.f / sqrtf(block_sum(ss, scratch) * inv_n + eps);
  const size_t orow = static_cast<size_t>(r_out) * hidden;
#pragma unroll
  for (int k = 0; k < ITEMS; ++k) {
    const int i = W * (tid + k * THREADS);
    if (i >= hidden) continue;
    if constexpr (VEC) {
      const float4 g = Vec4<float>::load(gain + i);
      float4 v = {(u[k][0] - mean) * inv * g.x, (u[k][1] - mean) * inv * g.y, (u[k][2] - mean) * inv * g.z,
                  (u[k][3] - mean) * inv * g.w};
      if (shift) v = add4(v, Vec4<float>::load(shift + i));
      Vec4<TO>::store(out + orow + i, v);
    } else {
      float v = (u[k][0] - mean) * inv * gain[i];
      if (shift) v += shift[i];
      out[orow + i] = from_float<TO>(v);
    }
  }
}

}  // namespace

extern "C" int pyre_stream_norm(const float* src, int src_streams, float* dst, int streams, const void* y, int y_dt,
                                int n_partials, long partial_stride, const float* mix, const float* out_w,
                                const float* in_w, const float* gain, const float* shift, int center, float eps, void* out,
                                int out_dt, const int* picked, int n, int hidden, hipStream_t stream) {
  PYRE_REQUIRE(streams >= 1 && streams <= kMaxStreams, "stream_norm: %d streams are outside 1..%d", streams, kMaxStreams);
  PYRE_REQUIRE(src && (src_streams == 1 || src_streams == streams), "stream_norm: the source has %d rows a token", src_streams);
  PYRE_REQUIRE(known_dtype(out_dt) && gain && out && hidden > 0 && eps > 0.f, "stream_norm: bad norm");
  PYRE_REQUIRE(!y || (known_dtype(y_dt) && n_partials >= 1 && mix && out_w), "stream_norm: a result needs partial sums, mix and out");
  PYRE_REQUIRE(hidden <= 16384, "stream_norm: rows of %d elements are more than 16384", hidden);
  if (n <= 0) return 0;
  const auto a16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = hidden % 4 == 0 && (!y || partial_stride % 4 == 0) && a16(src) && a16(dst) && a16(y) && a16(gain) && a16(shift) && a16(out);
#define PYRE_SN(S, THREADS, ITEMS, VEC)                                                                                     \
  hipLaunchKernelGGL((stream_norm_kernel<TD, TO, S, THREADS, ITEMS, VEC>), dim3(n), dim3(THREADS), 0, stream, src,          \
                     src_streams, dst, streams, static_cast<const TD*>(y), n_partials,                                      \
                     static_cast<size_t>(partial_stride), mix, out_w, in_w, gain, shift, center, eps,                       \
                     static_cast<TO*>(out), picked, hidden)
  // as for the other norms: which shape runs depends on the number of rows, what it computes does not but for the order
  // in which a row's block sum adds its threads; a few rows (a decode step) are spread over more threads each
#define PYRE_SN_SHAPE(S)                                            \
  do {                                                              \
    const int quads = hidden / 4;                                   \
    if (quads <= 256) PYRE_SN(S, 256, 1, true);                     \
    else if (n <= 128 && quads <= 1024) PYRE_SN(S, 1024, 1, true);  \
    else if (quads <= 1024) PYRE_SN(S, 256, 4, true);               \
    else PYRE_SN(S, 1024, 4, true);                                 \
  } while (0)
  PYRE_DISPATCH(y ? y_dt : kF32, TD, PYRE_DISPATCH(out_dt, TO, {
    if (!vec) {  // any width, any number of streams
      if (hidden <= 256) PYRE_SN(kMaxStreams, 256, 1, false);
      else if (hidden <= 4096) PYRE_SN(kMaxStreams, 1024, 4, false);
      else PYRE_SN(kMaxStreams, 1024, 16, false);
    } else if (streams <= 2) {
      PYRE_SN_SHAPE(2);
    } else if (streams <= 4) {
      PYRE_SN_SHAPE(4);
    } else if (hidden <= 4096) {
      PYRE_SN(kMaxStreams, 1024, 1, true);
    } else {
      PYRE_SN(kMaxStreams, 1024, 4, true);
    }
  }));
#undef PYRE_SN_SHAPE
#undef PYRE_SN
  return check_launch("stream_norm");
}
