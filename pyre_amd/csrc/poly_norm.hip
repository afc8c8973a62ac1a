// The polynomial activation with norms: act(z) = a N(z) + b N(z^2) + c N(z^3) + e over a token's row z of a product
// (its partial sums added first), where powers are element by element and N divides a row by its root mean square,
// sqrt(mean(.^2) + eps). Three sums over the row (of z^2, z^4 and z^6), then one polynomial per element with the
// norms folded into its coefficients. All arithmetic float32; one rounding at the store.
#include "pyre_api.h"
#include "pyre_common.h"
#include "pyre_vec4.h"

using namespace pyre;

namespace {

// z -> ((c3 z + c2) z + c1) z + c0: the coefficients with the norms in them.
struct Poly {
  float c0, c1, c2, c3;
  __device__ float operator()(float z) const { return fmaf(z, fmaf(z, fmaf(z, c3, c2), c1), c0); }
};

template <int THREADS>
__device__ inline Poly poly_of_row(float s2, float s4, float s6, const float* abce, float eps, int width, float* scratch) {
  const float inv_n = 1.f / static_cast<float>(width);
  // the three block sums with one barrier pair: every wave leaves its three sums, everybody adds them in order
  s2 = wave_sum(s2), s4 = wave_sum(s4), s6 = wave_sum(s6);
  const int w = threadIdx.x / kWave;
  constexpr int kWaves = THREADS / kWave;
  if (threadIdx.x % kWave == 0) scratch[w] = s2, scratch[kWaves + w] = s4, scratch[2 * kWaves + w] = s6;
  __syncthreads();
  s2 = s4 = s6 = 0.f;
#pragma unroll
  for (int i = 0; i < kWaves; ++i) s2 += scratch[i], s4 += scratch[kWaves + i], s6 += scratch[2 * kWaves + i];
  return Poly{abce[3], abce[0] / sqrtf(s2 * inv_n + eps), abce[1] / sqrtf(s4 * inv_n + eps), abce[2] / sqrtf(s6 * inv_n + eps)};
}

__device__ inline void add_powers(float z, float& s2, float& s4, float& s6) {
  const float q = z * z, r = q * q;
  s2 += q, s4 += r, s6 = fmaf(r, q, s6);
}

// A row in the block's registers: ITEMS groups of four elements a thread.
template <typename TI, typename TO, int THREADS, int ITEMS>
__global__ __launch_bounds__(THREADS) void poly_norm_vec_kernel(const TI* __restrict__ z, int n_partials, size_t partial_stride,
                                                                const float* __restrict__ abce, float eps,
                                                                TO* __restrict__ out, int width) {
  __shared__ float scratch[3 * THREADS / kWave];
  const size_t row = static_cast<size_t>(blockIdx.x) * width;
  float4 v[ITEMS];
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
#pragma unroll
  for (int k = 0; k < ITEMS; ++k) {
    const int i = 4 * (threadIdx.x + k * THREADS);
    v[k] = float4{0.f, 0.f, 0.f, 0.f};
    if (i < width) v[k] = n_partials == 1 ? Vec4<TI>::load(z + row + i) : sum_partials4(z + row + i, partial_stride, n_partials);
  }
#pragma unroll
  for (int k = 0; k < ITEMS; ++k) {
    add_powers(v[k].x, s2, s4, s6), add_powers(v[k].y, s2, s4, s6);
    add_powers(v[k].z, s2, s4, s6), add_powers(v[k].w, s2, s4, s6);
  }
  const Poly p = poly_of_row<THREADS>(s2, s4, s6, abce, eps, width, scratch);
#pragma unroll
  for (int k = 0; k < ITEMS; ++k) {
    const int i = 4 * (threadIdx.x + k * THREADS);
    if (i < width) Vec4<TO>::store(out + row + i, float4{p(v[k].x), p(v[k].y), p(v[k].z), p(v[k].w)});
  }
}

// Any width: the row is read twice.
template <typename TI, typename TO, int THREADS>
__global__ __launch_bounds__(THREADS) void poly_norm_kernel(const TI* __restrict__ z, int n_partials, size_t partial_stride,
                                                            const float* __restrict__ abce, float eps, TO* __restrict__ out,
                                                            int width) {
  __shared__ float scratch[3 * THREADS / kWave];
  const size_t row = static_cast<size_t>(blockIdx.x) * width;
  auto value = [&](int i) {
    float v = 0.f;
    for (int p = 0; p < n_partials; ++p) v += to_float(z[p * partial_stride + row + i]);
    return v;
  };
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  for (int i = threadIdx.x; i < width; i += THREADS) add_powers(value(i), s2, s4, s6);
  const Poly p = poly_of_row<THREADS>(s2, s4, s6, abce, eps, width, scratch);
  for (int i = threadIdx.x; i < width; i += THREADS) out[row + i] = from_float<TO>(p(value(i)));
}

}  // namespace

extern "C" int pyre_poly_norm(const void* z, int z_dt, int n_partials, long partial_stride, const float* abce, float eps,
                              void* out, int out_dt, int n, int width, hipStream_t stream) {
  PYRE_REQUIRE(known_dtype(z_dt) && known_dtype(out_dt) && n_partials >= 1 && abce, "poly_norm: bad arguments");
  PYRE_REQUIRE(width > 0 && eps > 0.f, "poly_norm: bad sizes");
  if (n <= 0) return 0;
  const bool vec = width % 4 == 0 && partial_stride % 4 == 0 && reinterpret_cast<uintptr_t>(z) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0 && width <= 4 * 1024 * 8;
  const int quads = width / 4;
#define PYRE_PN(THREADS, ITEMS)                                                                                           \
  hipLaunchKernelGGL((poly_norm_vec_kernel<TI, TO, THREADS, ITEMS>), dim3(n), dim3(THREADS), 0, stream,                   \
                     static_cast<const TI*>(z), n_partials, static_cast<size_t>(partial_stride), abce, eps,               \
                     static_cast<TO*>(out), width)
  PYRE_DISPATCH(z_dt, TI, PYRE_DISPATCH(out_dt, TO, {
    if (!vec)
      hipLaunchKernelGGL((poly_norm_kernel<TI, TO, 512>), dim3(n), dim3(512), 0, stream, static_cast<const TI*>(z), n_partials,
                         static_cast<size_t>(partial_stride), abce, eps, static_cast<TO*>(out), width);
    else if (quads <= 256) PYRE_PN(256, 1);
    else if (quads <= 1024) PYRE_PN(1024, 1);
    else if (quads <= 3072) PYRE_PN(1024, 3);
    else if (quads <= 5120) PYRE_PN(1024, 5);
    else PYRE_PN(1024, 8);
  }));
#undef PYRE_PN
  return check_launch("poly_norm");
}
