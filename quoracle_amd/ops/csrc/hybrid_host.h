// Host side that the hybrid-model modules share: argument checks, dispatch over
// activation types, and the wrappers of the stream kernels.  Included once by
// each module's binding file, inside its anonymous namespace.
#pragma once

using torch::Tensor;
using OptTensor = c10::optional<Tensor>;

hipStream_t current_stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

#define CHECK_GPU(t)                                                     \
  TORCH_CHECK((t).is_cuda(), #t " must be on the GPU");                  \
  TORCH_CHECK((t).is_contiguous(), #t " must be contiguous")
#define CHECK_I32(t)                                                     \
  CHECK_GPU(t);                                                          \
  TORCH_CHECK((t).scalar_type() == torch::kInt32, #t " must be int32")
#define CHECK_F32(t)                                                     \
  CHECK_GPU(t);                                                          \
  TORCH_CHECK((t).scalar_type() == torch::kFloat32, #t " must be float32")

template <typename T> constexpr torch::ScalarType scalar_of();
template <> constexpr torch::ScalarType scalar_of<bf16>() {
  return torch::kBFloat16;
}
template <> constexpr torch::ScalarType scalar_of<float>() {
  return torch::kFloat32;
}
template <typename T> T *ptr(const Tensor &t) {
  TORCH_CHECK(t.scalar_type() == scalar_of<T>(), "mixed activation dtypes");
  return reinterpret_cast<T *>(t.data_ptr());
}
const int *iptr(const Tensor &t) { return t.data_ptr<int>(); }
float *fptr(const Tensor &t) { return t.data_ptr<float>(); }

// Run `body` with T = the activation type of `t`.
template <typename F> void by_dtype(const Tensor &t, F body) {
  if (t.scalar_type() == torch::kBFloat16) body(bf16());
  else if (t.scalar_type() == torch::kFloat32) body(float());
  else TORCH_CHECK(false, "activations must be bfloat16 or float32");
}
template <int N> using Int = std::integral_constant<int, N>;
template <typename F> void by_vec(bool vec8, F body) {
  if (vec8) body(Int<8>());
  else body(Int<1>());
}
// Register groups per thread of a 256-thread norm over n values; 0: too many.
template <typename F> void by_items(int n, int vec, F body) {
  const int need = (n + 256 * vec - 1) / (256 * vec);
  if (need <= 1) body(Int<1>());
  else if (need <= 2) body(Int<2>());
  else if (need <= 4) body(Int<4>());
  else body(Int<0>());
}

void embed_positions(Tensor x, Tensor h, Tensor embed, OptTensor table,
                     Tensor tokens, Tensor positions) {
  CHECK_F32(x); CHECK_GPU(h); CHECK_GPU(embed);
  CHECK_I32(tokens); CHECK_I32(positions);
  const int n = embed.size(1);
  const long T = tokens.size(0);
  TORCH_CHECK(x.numel() == T * n && h.numel() == T * n &&
              positions.size(0) == T, "embed_positions shapes");
  if (table) { CHECK_GPU(*table); TORCH_CHECK(table->size(1) == n, "table"); }
  if (T == 0) return;
  by_dtype(embed, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      embed_positions_kernel<A, decltype(v)::value>
          <<<dim3(T), dim3(256), 0, current_stream()>>>(
              fptr(x), ptr<A>(h), ptr<A>(embed),
              table ? ptr<A>(*table) : nullptr, iptr(tokens), iptr(positions),
              n);
    });
  });
  HIP_CHECK_KERNEL();
}

void norm_rows(Tensor out, Tensor x, Tensor rows, Tensor w, double eps) {
  CHECK_GPU(out); CHECK_F32(x); CHECK_GPU(rows); CHECK_F32(w);
  TORCH_CHECK(rows.scalar_type() == torch::kInt64, "rows must be int64");
  const int n = w.size(0);
  const long R = rows.size(0);
  TORCH_CHECK(out.numel() == R * n && x.size(-1) == n, "norm_rows shapes");
  if (R == 0) return;
  by_dtype(out, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      norm_rows_kernel<A, decltype(v)::value>
          <<<dim3(R), dim3(256), 0, current_stream()>>>(
              ptr<A>(out), fptr(x),
              reinterpret_cast<const long *>(rows.data_ptr<int64_t>()),
              fptr(w), n, (float)eps);
    });
  });
  HIP_CHECK_KERNEL();
}

void pre_norm(Tensor x, Tensor h, OptTensor y, Tensor w, double eps) {
  CHECK_F32(x); CHECK_GPU(h); CHECK_F32(w);
  const int n = w.size(0);
  const long T = x.numel() / n;
  TORCH_CHECK(x.numel() == T * n && h.numel() == T * n, "pre_norm shapes");
  if (y) { CHECK_F32(*y); TORCH_CHECK(y->numel() == T * n, "pre_norm y"); }
  if (T == 0) return;
  by_dtype(h, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      pre_norm_kernel<A, decltype(v)::value>
          <<<dim3(T), dim3(256), 0, current_stream()>>>(
              fptr(x), ptr<A>(h), y ? fptr(*y) : nullptr, fptr(w), n,
              (float)eps);
    });
  });
  HIP_CHECK_KERNEL();
}

// a w^T with a float32 result.
Tensor linear_f32(const Tensor &a, const Tensor &w) {
  if (a.scalar_type() == torch::kFloat32) return at::linear(a, w);
  return at::mm(a, w.t(), torch::kFloat32);
}
