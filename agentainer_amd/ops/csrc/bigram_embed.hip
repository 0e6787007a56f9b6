// Token embeddings (gfx950).
//
// embed_rows: the table's rows as the fp32 stream, and as they are into a
// column range of a wider matrix (the input of a projection that reads the
// embedding again).
//
// With a second table:
//
// position_embed_norm: x[r] = rms_norm(scale * embed[id_r] + pos[p_r]) * w,
// fp32 out, optionally written twice (the second copy is what later passes
// of a repeated layer group add again). One workgroup per row; the sum stays
// in registers between the two passes.
//
// bigram_embed: scaled token embedding plus a hashed bigram embedding
//
//   x[r] = scale * embed[id_r] + bigram[row_r]            (fp32 out)
//   row_r = (mul_prev * id_(r-1) + mul_cur * id_r) mod buckets,
//   row_r = buckets (the table's last row) for a sequence's first token.
//
// The previous id of a step's first row of a sequence is per-sequence state
// (prev_state[slot], int32); a sequence whose first row sits at position 0
// ignores it. Kernel 1 (one workgroup per token row) only READS the state;
// kernel 2 (one thread per sequence) then stores the portion's last id, so
// rows of one sequence that run in different workgroups never race with
// the update.

#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include "latent_common.h"

namespace {

__device__ __forceinline__ int find_seq(const int* starts, int B, int t) {
  int lo = 0, hi = B - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (starts[mid] <= t) lo = mid; else hi = mid - 1;
  }
  return lo;
}

template <typename T>
__global__ __launch_bounds__(256) void bigram_embed_kernel(
    float* __restrict__ x, const long* __restrict__ ids,
    const T* __restrict__ embed, const T* __restrict__ bigram, float scale,
    long mul_prev, long mul_cur, long buckets,
    const int* __restrict__ prev_state, const long* __restrict__ slots,
    const int* __restrict__ seq_lens, const int* __restrict__ q_starts,
    const int* __restrict__ q_lens, int B, int W, long vocab) {
  const int r = blockIdx.x;
  long id = ids[r];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* er = embed + id * W;
  const T* br = nullptr;
  if (bigram != nullptr) {
    int b, off, n;
    if (q_starts) {
      b = find_seq(q_starts, B, r);
      off = r - q_starts[b];
      n = q_lens[b];
    } else {
      b = r; off = 0; n = 1;
    }
    const int pos = seq_lens[b] - n + off;
    long row = buckets;
    if (pos > 0) {
      const long prev = off > 0 ? ids[r - 1] : (long)prev_state[slots[b]];
      row = (prev * mul_prev + id * mul_cur) % buckets;
      if (row < 0) row += buckets;
    }
    br = bigram + row * W;
  }
  float* xr = x + (long)r * W;
  if (W % 4 == 0) {   // table rows then start 4-element aligned
    for (int i = threadIdx.x * 4; i < W; i += 256 * 4) {
      float v[4], b[4] = {0.f, 0.f, 0.f, 0.f};
      ld4(er, i, v);
      if (br) ld4(br, i, b);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = fmaf(v[j], scale, b[j]);
      st4(xr, i, v);
    }
    return;
  }
  for (int i = threadIdx.x; i < W; i += 256) {
    float v = ldf(er, i) * scale;
    if (br) v += ldf(br, i);
    xr[i] = v;
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void embed_rows_kernel(
    float* __restrict__ x, T* __restrict__ raw, long raw_rs,
    const long* __restrict__ ids, const T* __restrict__ embed, int W,
    long vocab) {
  const long r = blockIdx.x;
  long id = ids[r];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  for (int i = threadIdx.x * VEC; i < W; i += 256 * VEC) {
    float v[VEC];
    if constexpr (VEC == 4) {
      ld4(embed, id * W + i, v);
      if (x) st4(x, r * W + i, v);
      if (raw) st4(raw, r * raw_rs + i, v);
    } else {
      v[0] = ldf(embed, id * W + i);
      if (x) x[r * W + i] = v[0];
      if (raw) stf(raw, r * raw_rs + i, v[0]);
    }
  }
}

__global__ void bigram_state_kernel(int* __restrict__ prev_state,
                                    const long* __restrict__ ids,
                                    const long* __restrict__ slots,
                                    const int* __restrict__ q_starts,
                                    const int* __restrict__ q_lens, int B) {
  const int b = blockIdx.x * blockDim.x + threadIdx.x;
  if (b >= B) return;
  const int n = q_lens ? q_lens[b] : 1;
  if (n <= 0) return;
  const int last = (q_starts ? q_starts[b] : b) + n - 1;
  prev_state[slots[b]] = (int)ids[last];
}

constexpr int ROW_VALS = 32;   // values per thread: rows of up to 8192

// NV groups of VEC consecutive values per thread hold the row
template <typename T, int VEC, int NV>
__global__ __launch_bounds__(256) void position_embed_kernel(
    float* __restrict__ x, float* __restrict__ x_copy,
    const long* __restrict__ ids, const int* __restrict__ positions,
    const T* __restrict__ embed, const T* __restrict__ pos, float scale,
    const float* __restrict__ w, float eps, int W, long vocab, int n_pos) {
  __shared__ float red[4];
  const long r = blockIdx.x;
  long id = ids[r];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  int p = positions[r];
  p = p < 0 ? 0 : (p >= n_pos ? n_pos - 1 : p);
  const T* er = embed + id * W;
  const T* pr = pos + (long)p * W;
  float v[NV][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int i = (k * 256 + threadIdx.x) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[k][j] = 0.f;
    if (i < W) {
      float p4[VEC];
      if constexpr (VEC == 4) {
        ld4(er, i, v[k]);
        ld4(pr, i, p4);
      } else {
        v[k][0] = ldf(er, i);
        p4[0] = ldf(pr, i);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        v[k][j] = fmaf(v[k][j], scale, p4[j]);
        ss = fmaf(v[k][j], v[k][j], ss);
      }
    }
  }
  const float rs = 1.0f / sqrtf(block_sum_256(ss, red) / (float)W + eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int i = (k * 256 + threadIdx.x) * VEC;
    if (i < W) {
      float wv[VEC];
      if constexpr (VEC == 4) ld4(w, i, wv); else wv[0] = w[i];
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[k][j] *= rs * wv[j];
      if constexpr (VEC == 4) {
        st4(x, r * W + i, v[k]);
        if (x_copy) st4(x_copy, r * W + i, v[k]);
      } else {
        x[r * W + i] = v[k][0];
        if (x_copy) x_copy[r * W + i] = v[k][0];
      }
    }
  }
}

}  // namespace

void embed_rows(c10::optional<torch::Tensor> x,
                c10::optional<torch::Tensor> raw, torch::Tensor ids,
                torch::Tensor embed) {
  TORCH_CHECK(ids.scalar_type() == at::kLong && ids.is_contiguous());
  TORCH_CHECK(embed.dim() == 2 && embed.is_contiguous() && embed.size(0) >= 1);
  const int T_ = ids.numel(), W = embed.size(1);
  float* xp = nullptr;
  void* rp = nullptr;
  long raw_rs = 0;
  bool vec = W % 4 == 0;
  if (x.has_value()) {
    TORCH_CHECK(x->scalar_type() == at::kFloat && x->is_contiguous() &&
                x->dim() == 2 && x->size(0) == T_ && x->size(1) == W);
    xp = x->data_ptr<float>();
  }
  if (raw.has_value()) {
    TORCH_CHECK(raw->scalar_type() == embed.scalar_type() && raw->dim() == 2 &&
                raw->size(0) == T_ && raw->size(1) == W &&
                raw->stride(1) == 1);
    rp = raw->data_ptr();
    raw_rs = raw->stride(0);
    vec = vec && raw_rs % 4 == 0 && raw->storage_offset() % 4 == 0;
  }
  if (T_ == 0 || (!xp && !rp)) return;
  auto stream = at::hip::getCurrentHIPStream();
#define LAUNCH(V)                                                             \
  hipLaunchKernelGGL((embed_rows_kernel<T, V>), dim3(T_), dim3(256), 0,       \
                     stream, xp, (T*)rp, raw_rs, ids.data_ptr<long>(),        \
                     (const T*)embed.data_ptr(), W, (long)embed.size(0))
  LATENT_DISPATCH_T(embed, {
    if (vec) LAUNCH(4); else LAUNCH(1);
  });
#undef LAUNCH
}

void position_embed_norm(torch::Tensor x, c10::optional<torch::Tensor> x_copy,
                         torch::Tensor ids, torch::Tensor positions,
                         torch::Tensor embed, torch::Tensor pos, double scale,
                         torch::Tensor w, double eps) {
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.is_contiguous() &&
              x.dim() == 2);
  const int T_ = x.size(0), W = x.size(1);
  TORCH_CHECK(W <= 256 * ROW_VALS, "row wider than ", 256 * ROW_VALS);
  TORCH_CHECK(ids.scalar_type() == at::kLong && ids.is_contiguous() &&
              ids.numel() == T_);
  TORCH_CHECK(positions.scalar_type() == at::kInt &&
              positions.is_contiguous() && positions.numel() == T_);
  TORCH_CHECK(embed.dim() == 2 && embed.is_contiguous() && embed.size(1) == W);
  TORCH_CHECK(pos.dim() == 2 && pos.is_contiguous() && pos.size(1) == W &&
              pos.size(0) >= 1 && pos.scalar_type() == embed.scalar_type());
  TORCH_CHECK(w.scalar_type() == at::kFloat && w.is_contiguous() &&
              w.numel() == W);
  float* xc = nullptr;
  if (x_copy.has_value()) {
    TORCH_CHECK(x_copy->scalar_type() == at::kFloat &&
                x_copy->is_contiguous() && x_copy->sizes() == x.sizes());
    xc = x_copy->data_ptr<float>();
  }
  if (T_ == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
#define LAUNCH(V, N)                                                          \
  hipLaunchKernelGGL((position_embed_kernel<T, V, N>), dim3(T_), dim3(256), 0,\
                     stream, x.data_ptr<float>(), xc, ids.data_ptr<long>(),   \
                     positions.data_ptr<int>(), (const T*)embed.data_ptr(),   \
                     (const T*)pos.data_ptr(), (float)scale,                  \
                     w.data_ptr<float>(), (float)eps, W, (long)embed.size(0), \
                     (int)pos.size(0))
  LATENT_DISPATCH_T(embed, {
    if (W % 4 == 0) {
      if (W <= 256 * 4 * 2) LAUNCH(4, 2);
      else if (W <= 256 * 4 * 4) LAUNCH(4, 4);
      else LAUNCH(4, ROW_VALS / 4);
    } else {
      LAUNCH(1, ROW_VALS);
    }
  });
#undef LAUNCH
}

void bigram_embed(torch::Tensor x, torch::Tensor ids, torch::Tensor embed,
                  c10::optional<torch::Tensor> bigram, double scale,
                  long mul_prev, long mul_cur, long buckets,
                  c10::optional<torch::Tensor> prev_state,
                  torch::Tensor state_slots, torch::Tensor seq_lens,
                  c10::optional<torch::Tensor> query_starts,
                  c10::optional<torch::Tensor> query_lens) {
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.is_contiguous() &&
              x.dim() == 2);
  const int T_ = x.size(0), W = x.size(1);
  TORCH_CHECK(ids.scalar_type() == at::kLong && ids.is_contiguous() &&
              ids.numel() == T_);
  TORCH_CHECK(embed.dim() == 2 && embed.is_contiguous() && embed.size(1) == W);
  TORCH_CHECK(seq_lens.scalar_type() == at::kInt && seq_lens.is_contiguous());
  const int B = seq_lens.numel();
  TORCH_CHECK(state_slots.scalar_type() == at::kLong &&
              state_slots.is_contiguous() && state_slots.numel() == B);
  TORCH_CHECK(query_starts.has_value() == query_lens.has_value());
  const int* qs = nullptr;
  const int* ql = nullptr;
  if (query_starts.has_value()) {
    TORCH_CHECK(query_starts->scalar_type() == at::kInt &&
                query_lens->scalar_type() == at::kInt &&
                query_starts->numel() == B && query_lens->numel() == B &&
                query_starts->is_contiguous() && query_lens->is_contiguous());
    qs = query_starts->data_ptr<int>();
    ql = query_lens->data_ptr<int>();
  } else {
    TORCH_CHECK(T_ == B, "decode: one row per sequence");
  }
  const void* bp = nullptr;
  int* ps = nullptr;
  if (bigram.has_value()) {
    TORCH_CHECK(bigram->dim() == 2 && bigram->is_contiguous() &&
                bigram->size(1) == W && bigram->size(0) == buckets + 1 &&
                bigram->scalar_type() == embed.scalar_type() && buckets >= 1,
                "bigram table must hold buckets + 1 rows");
    TORCH_CHECK(prev_state.has_value() &&
                prev_state->scalar_type() == at::kInt &&
                prev_state->is_contiguous(),
                "a bigram table needs the int32 previous-token state");
    bp = bigram->data_ptr();
    ps = prev_state->data_ptr<int>();
  }
  if (T_ == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  LATENT_DISPATCH_T(embed, {
    hipLaunchKernelGGL((bigram_embed_kernel<T>), dim3(T_), dim3(256), 0,
                       stream, x.data_ptr<float>(), ids.data_ptr<long>(),
                       (const T*)embed.data_ptr(), (const T*)bp, (float)scale,
                       mul_prev, mul_cur, buckets, ps,
                       state_slots.data_ptr<long>(), seq_lens.data_ptr<int>(),
                       qs, ql, B, W, (long)embed.size(0));
  });
  if (ps != nullptr)
    hipLaunchKernelGGL(bigram_state_kernel, dim3((B + 63) / 64), dim3(64), 0,
                       stream, ps, ids.data_ptr<long>(),
                       state_slots.data_ptr<long>(), qs, ql, B);
}
