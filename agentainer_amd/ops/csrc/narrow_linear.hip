// Narrow projections with an fp32 result (gfx950): routers, decay and
// write-strength projections.
//
//   out[t, n] = sum_k x[t, k] * w[n, k] + bias[n]      x, w bf16; out fp32
//
// Products of bf16 values are exact in fp32 and the sum is kept in fp32, so
// the result is the 32-bit projection of the bf16 rows; a library bf16 GEMM
// would round it to bf16 and a library fp32 GEMM first needs fp32 copies of
// the (wide) rows.
//
// A workgroup of 8 waves owns RT 16-row and NT 16-column tiles. The waves cut
// K among themselves in interleaved steps of 32 (together they walk whole
// 512-byte stretches of every row), each feeds v_mfma_f32_16x16x32_bf16
// straight from global memory — there is nothing to share through LDS but
// the eight partial sums at the end. Wide steps take NT = 4 (every row is
// read once per 64 columns), short ones NT = 1 so that a decode step still
// spreads over the columns. Many rows with many columns take RT = 2 or 4:
// every weight fragment then serves that many row tiles (with one, the
// workgroups' reads of the weights are what bounds the kernel). The order of
// a row's sum depends on none of this.
//
// MFMA fragment maps (v_mfma_f32_16x16x32_bf16): A lane l holds
// A[l%16][(l/16)*8 + j]; B lane l holds B[(l/16)*8 + j][l%16]; C/D lane l
// holds rows (l/16)*4 + r, column l%16.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include "latent_common.h"

namespace {

typedef __bf16 bf16v8 __attribute__((ext_vector_type(8)));

constexpr int NW = 8;       // waves of a workgroup
constexpr int KSTEP = 32;
constexpr int UNROLL = 4;   // K steps whose loads are in flight together

// 8 consecutive values of a row from column k; past the end: zeros
template <bool VEC>
__device__ __forceinline__ bf16v8 row8(const short* p, int k, int K) {
  bf16x8 v{};
  if constexpr (VEC) {
    if (k < K) v = *reinterpret_cast<const bf16x8*>(p + k);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (k + j < K) v[j] = p[k + j];
  }
  bf16v8 r;
  __builtin_memcpy(&r, &v, 16);
  return r;
}

template <int NT, int RT, bool VEC>
__global__ __launch_bounds__(NW * 64) void narrow_linear_kernel(
    float* __restrict__ out, const short* __restrict__ x, long x_rs,
    const short* __restrict__ w, const float* __restrict__ bias, int T, int N,
    int K) {
  __shared__ float part[NW][NT][16 * 17];
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int l16 = lane & 15, lg = lane >> 4;
  const int t0 = blockIdx.x * 16 * RT, n0 = blockIdx.y * (16 * NT);
  // rows and columns past the end are clamped: loaded, never stored
  const short* xp[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i)
    xp[i] = x + (long)min(t0 + i * 16 + l16, T - 1) * x_rs;
  const short* wp[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
    wp[i] = w + (long)min(n0 + i * 16 + l16, N - 1) * K;
  f32x4 acc[RT][NT];
#pragma unroll
  for (int m = 0; m < RT; ++m)
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[m][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int UN = RT == 4 ? UNROLL / 2 : UNROLL;
  for (int k0 = wid * KSTEP; k0 < K; k0 += NW * KSTEP * UN) {
    bf16v8 a[UN][RT], b[UN][NT];
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int k = k0 + u * NW * KSTEP + lg * 8;
#pragma unroll
      for (int m = 0; m < RT; ++m) a[u][m] = row8<VEC>(xp[m], k, K);
#pragma unroll
      for (int i = 0; i < NT; ++i) b[u][i] = row8<VEC>(wp[i], k, K);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u)
#pragma unroll
      for (int m = 0; m < RT; ++m)
#pragma unroll
        for (int i = 0; i < NT; ++i)
          acc[m][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              a[u][m], b[u][i], acc[m][i], 0, 0, 0);
  }
#pragma unroll
  for (int m = 0; m < RT; ++m) {
    if (m > 0) __syncthreads();        // the previous tile's sums are read
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        part[wid][i][(lg * 4 + r) * 17 + l16] = acc[m][i][r];
    __syncthreads();
    for (int e = threadIdx.x; e < NT * 256; e += NW * 64) {
      const int i = e >> 8, r = (e >> 4) & 15, c = e & 15;
      const int t = t0 + m * 16 + r, n = n0 + i * 16 + c;
      if (t < T && n < N) {
        float s = 0.f;
#pragma unroll
        for (int q = 0; q < NW; ++q) s += part[q][i][r * 17 + c];
        out[(long)t * N + n] = s + (bias ? bias[n] : 0.f);
      }
    }
  }
}

}  // namespace

void narrow_linear(torch::Tensor out, torch::Tensor x, torch::Tensor w,
                   c10::optional<torch::Tensor> bias) {
  TORCH_CHECK(x.dim() == 2 && x.stride(1) == 1 &&
              x.scalar_type() == at::kBFloat16);
  TORCH_CHECK(w.dim() == 2 && w.is_contiguous() &&
              w.scalar_type() == at::kBFloat16 && w.size(1) == x.size(1));
  const int T_ = x.size(0), K = x.size(1), N = w.size(0);
  TORCH_CHECK(out.scalar_type() == at::kFloat && out.is_contiguous() &&
              out.dim() == 2 && out.size(0) == T_ && out.size(1) == N);
  const float* bp = nullptr;
  if (bias.has_value()) {
    TORCH_CHECK(bias->scalar_type() == at::kFloat && bias->is_contiguous() &&
                bias->numel() == N);
    bp = bias->data_ptr<float>();
  }
  if (T_ == 0 || N == 0) return;
  TORCH_CHECK(K >= 1);
  const bool vec = K % 8 == 0 && x.stride(0) % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(x.data_ptr()) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(w.data_ptr()) % 16 == 0;
  const int tb = (T_ + 15) / 16;
  auto stream = at::hip::getCurrentHIPStream();
#define LAUNCH(NT, RT, V)                                                     \
  hipLaunchKernelGGL((narrow_linear_kernel<NT, RT, V>),                       \
                     dim3((tb + RT - 1) / RT, (N + 16 * NT - 1) / (16 * NT)), \
                     dim3(NW * 64), 0, stream, out.data_ptr<float>(),                        \
                     (const short*)x.data_ptr(), (long)x.stride(0),           \
                     (const short*)w.data_ptr(), bp, T_, N, K)
  // row tiles: as many as leave the chip 256 workgroups
  const long wide = (long)tb * ((N + 63) / 64);
  if (!vec) LAUNCH(1, 1, false);
  else if (N <= 16 || tb < 128) LAUNCH(1, 1, true);
  else if (N <= 32) LAUNCH(2, 1, true);
  else if (wide < 512) LAUNCH(4, 1, true);
  else if (wide < 1024) LAUNCH(4, 2, true);
  else LAUNCH(4, 4, true);
#undef LAUNCH
}
