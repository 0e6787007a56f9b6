// Query / key norm over ALL heads of a token at once, query temperature and
// the paged K/V append (gfx950).
//
//   q [T, H*D]  <- q / sqrt(mean(q^2) + eps) * q_w * temp(p)      (in place)
//   k [T, G*D]  -> k / sqrt(mean(k^2) + eps) * k_w                -> k_cache
//   v [T, G*Dv] -> v_cache as it is
//   temp(p) = 1 + coef * ln(floor((p + 1) / every) + 1),  p the position
//
// The means run over the whole row, before it is cut into heads. Pools are
// [P, G, PS, D] / [P, G, PS, Dv]; slot < 0 skips the append. All math is
// fp32. Two workgroups per token: one takes the query row, one the key row
// and the value copy. A row stays in registers between its sum and its store
// (NREG groups of VEC values per thread); rows too wide for that are read
// again (NREG = 0).

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include "latent_common.h"

namespace {

template <int VEC>
__device__ __forceinline__ void load_vec(const short* p, long i, float* v) {
  if constexpr (VEC == 8) {
    const bf16x8 t = *reinterpret_cast<const bf16x8*>(p + i);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = bits2f(t[j]);
  } else if constexpr (VEC == 4) {
    ld4(p, i, v);
  } else {
    v[0] = ldf(p, i);
  }
}
template <int VEC>
__device__ __forceinline__ void load_vec(const float* p, long i, float* v) {
  if constexpr (VEC >= 4) {
#pragma unroll
    for (int j = 0; j < VEC; j += 4) ld4(p, i + j, v + j);
  } else {
    v[0] = p[i];
  }
}
template <int VEC>
__device__ __forceinline__ void store_vec(short* p, long i, const float* v) {
  if constexpr (VEC == 8) {
    bf16x8 t;
#pragma unroll
    for (int j = 0; j < 8; ++j) t[j] = f2bits(v[j]);
    *reinterpret_cast<bf16x8*>(p + i) = t;
  } else if constexpr (VEC == 4) {
    st4(p, i, v);
  } else {
    stf(p, i, v[0]);
  }
}
template <int VEC>
__device__ __forceinline__ void store_vec(float* p, long i, const float* v) {
  if constexpr (VEC >= 4) {
#pragma unroll
    for (int j = 0; j < VEC; j += 4) st4(p, i + j, v + j);
  } else {
    p[i] = v[0];
  }
}

template <typename T, int VEC, int NREG>
__global__ __launch_bounds__(256) void row_norm_append_kernel(
    T* __restrict__ q, long q_rs, const T* __restrict__ k, long k_rs,
    const T* __restrict__ v, long v_rs, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const int* __restrict__ positions,
    const long* __restrict__ slots, float eps, const float* __restrict__ q_w,
    const float* __restrict__ k_w, float coef, int every, int nq, int G, int D,
    int Dv, int PS) {
  __shared__ float red[4];
  const long t = blockIdx.x;
  const bool is_q = blockIdx.y == 0;
  const long slot = is_q ? 0 : slots[t];
  if (slot < 0) return;                               // the whole workgroup
  const T* src = is_q ? q + t * q_rs : k + t * k_rs;
  const float* w = is_q ? q_w : k_w;
  const int n = is_q ? nq : G * D;
  constexpr int STEP = 256 * VEC;
  const int i0 = threadIdx.x * VEC;
  float x[NREG > 0 ? NREG : 1][VEC];
  float ss = 0.f;
  if constexpr (NREG > 0) {
#pragma unroll
    for (int r = 0; r < NREG; ++r) {
      const int i = i0 + r * STEP;
      if (i < n) {
        load_vec<VEC>(src, i, x[r]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss = fmaf(x[r][j], x[r][j], ss);
      }
    }
  } else {
    for (int i = i0; i < n; i += STEP) {
      load_vec<VEC>(src, i, x[0]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(x[0][j], x[0][j], ss);
    }
  }
  float mul = 1.0f / sqrtf(block_sum_256(ss, red) / (float)n + eps);
  if (is_q && coef != 0.f)
    mul *= fmaf(coef, logf((float)((positions[t] + 1) / every + 1)), 1.0f);
  T* kd = k_cache + ((slot / PS) * G * PS + slot % PS) * D;   // head 0
  auto put = [&](int i, const float* xv) {
    float wv[VEC], o[VEC];
    load_vec<VEC>(w, i, wv);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = xv[j] * mul * wv[j];
    if (is_q)
      store_vec<VEC>(q + t * q_rs, i, o);
    else
      store_vec<VEC>(kd + (long)(i / D) * PS * D, i % D, o);
  };
  if constexpr (NREG > 0) {
#pragma unroll
    for (int r = 0; r < NREG; ++r)
      if (i0 + r * STEP < n) put(i0 + r * STEP, x[r]);
  } else {
    for (int i = i0; i < n; i += STEP) {
      load_vec<VEC>(src, i, x[0]);
      put(i, x[0]);
    }
  }
  if (is_q) return;
  T* vd = v_cache + ((slot / PS) * G * PS + slot % PS) * Dv;
  for (int i = i0; i < G * Dv; i += STEP) {
    float o[VEC];
    load_vec<VEC>(v + t * v_rs, i, o);
    store_vec<VEC>(vd + (long)(i / Dv) * PS * Dv, i % Dv, o);
  }
}

}  // namespace

void row_norm_append(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                     torch::Tensor k_cache, torch::Tensor v_cache,
                     torch::Tensor positions, torch::Tensor slot_mapping,
                     double eps, torch::Tensor q_w, torch::Tensor k_w,
                     double temp_coef, long temp_every) {
  TORCH_CHECK(q.dim() == 2 && k.dim() == 2 && v.dim() == 2 &&
              q.stride(1) == 1 && k.stride(1) == 1 && v.stride(1) == 1);
  const int T_ = q.size(0), nq = q.size(1);
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.is_contiguous() &&
              v_cache.dim() == 4 && v_cache.is_contiguous());
  const int G = k_cache.size(1), PS = k_cache.size(2), D = k_cache.size(3);
  const int Dv = v_cache.size(3);
  TORCH_CHECK(v_cache.size(0) == k_cache.size(0) && v_cache.size(1) == G &&
              v_cache.size(2) == PS, "pool shapes disagree");
  TORCH_CHECK(k.size(0) == T_ && v.size(0) == T_ &&
              k.size(1) == (long)G * D && v.size(1) == (long)G * Dv &&
              nq >= 1 && nq % D == 0, "q/k/v rows do not fit the pools");
  TORCH_CHECK(k.scalar_type() == q.scalar_type() &&
              v.scalar_type() == q.scalar_type() &&
              k_cache.scalar_type() == q.scalar_type() &&
              v_cache.scalar_type() == q.scalar_type(),
              "q, k, v and the pools share one element type");
  TORCH_CHECK(positions.scalar_type() == at::kInt && positions.numel() == T_ &&
              positions.is_contiguous());
  TORCH_CHECK(slot_mapping.scalar_type() == at::kLong &&
              slot_mapping.numel() == T_ && slot_mapping.is_contiguous());
  TORCH_CHECK(q_w.scalar_type() == at::kFloat && q_w.is_contiguous() &&
              q_w.numel() == nq && k_w.scalar_type() == at::kFloat &&
              k_w.is_contiguous() && k_w.numel() == (long)G * D);
  TORCH_CHECK(temp_every >= 1, "temperature step must be positive");
  if (T_ == 0) return;
  // rows that start and end on multiples of n elements, heads likewise
  auto fits = [&](int n) {
    auto ok = [&](const torch::Tensor& t, long row) {
      const long bytes = n * (long)t.element_size();
      return row % n == 0 && reinterpret_cast<uintptr_t>(t.data_ptr()) %
                                     (bytes < 16 ? bytes : 16) == 0;
    };
    return D % n == 0 && Dv % n == 0 && ok(q, q.stride(0)) &&
           ok(k, k.stride(0)) && ok(v, v.stride(0)) && ok(k_cache, D) &&
           ok(v_cache, Dv) && ok(q_w, nq) && ok(k_w, D);
  };
  const int vec = fits(8) ? 8 : fits(4) ? 4 : 1;
  const int widest = nq > G * D ? nq : G * D;
  const int nreg = (widest + 256 * vec - 1) / (256 * vec);
  auto stream = at::hip::getCurrentHIPStream();
#define LAUNCH(V, N)                                                          \
  hipLaunchKernelGGL((row_norm_append_kernel<T, V, N>), dim3(T_, 2),          \
                     dim3(256), 0, stream, (T*)q.data_ptr(),                  \
                     (long)q.stride(0), (const T*)k.data_ptr(),               \
                     (long)k.stride(0), (const T*)v.data_ptr(),               \
                     (long)v.stride(0), (T*)k_cache.data_ptr(),               \
                     (T*)v_cache.data_ptr(), positions.data_ptr<int>(),       \
                     slot_mapping.data_ptr<long>(), (float)eps,               \
                     q_w.data_ptr<float>(), k_w.data_ptr<float>(),            \
                     (float)temp_coef, (int)temp_every, nq, G, D, Dv, PS)
#define LAUNCH_N(V)                                                           \
  do {                                                                        \
    if (nreg <= 1) LAUNCH(V, 1);                                              \
    else if (nreg == 2) LAUNCH(V, 2);                                         \
    else if (nreg <= 4) LAUNCH(V, 4);                                         \
    else LAUNCH(V, 0);                                                        \
  } while (0)
  LATENT_DISPATCH_T(q, {
    if (vec == 8) LAUNCH_N(8);
    else if (vec == 4) LAUNCH_N(4);
    else LAUNCH_N(1);
  });
#undef LAUNCH
#undef LAUNCH_N
}
