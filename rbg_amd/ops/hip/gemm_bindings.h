// Binding of the decode-shape GEMM, for every extension that links
// skinny_gemm.hip.
#pragma once
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include <hip/hip_runtime.h>

extern "C" {
void launch_skinny_gemm(void*, void*, const void*, const void*, int, int,
                        int, int, hipStream_t);
void launch_reduce_splits(void*, const void*, int, long, hipStream_t);
}

inline hipStream_t gemm_stream() {
  return at::hip::getCurrentHIPStream().stream();
}

inline int pick_gemm_splits(int N, int K) {
  // fill the chip with 16-wave workgroups (>= ~256 WGs); each split's K
  // range divides into 8 x 32-k wave slices (K % (splits*256) == 0)
  const int n_groups = N >> 5;
  for (int s : {8, 4, 2})
    if (n_groups * s <= 512 && n_groups * s >= 192 && K % (s * 256) == 0)
      return s;
  for (int s : {4, 2})
    if (n_groups * s >= 128 && K % (s * 256) == 0) return s;
  return 1;
}

inline bool skinny_gemm_supported(int64_t M, int64_t N, int64_t K) {
  // M <= 256: the cross-slice LDS reduce holds 4 waves x M_TILES x 1 KB
  // (64 KB at M_TILES=16); larger batches fall back to hipBLASLt
  return M >= 1 && M <= 256 && (N % 32) == 0 && (K % 256) == 0;
}

inline torch::Tensor skinny_gemm(torch::Tensor a, torch::Tensor w,
                          int64_t force_splits = 0) {
  for (const auto& t : {a, w})
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kBFloat16 &&
                t.is_contiguous() && t.dim() == 2,
                "operands must be contiguous bf16 matrices on GPU");
  const int64_t M = a.size(0), K = a.size(1), N = w.size(0);
  TORCH_CHECK(w.size(1) == K, "K mismatch");
  TORCH_CHECK(skinny_gemm_supported(M, N, K), "unsupported skinny shape");
  auto c = torch::empty({M, N}, a.options());
  int splits = force_splits > 0 ? (int)force_splits
                                : pick_gemm_splits((int)N, (int)K);
  if (K % (splits * 256) != 0) splits = pick_gemm_splits((int)N, (int)K);
  torch::Tensor ws;
  void* wsp = nullptr;
  if (splits > 1) {
    ws = torch::empty({splits, M, N}, a.options().dtype(torch::kFloat32));
    wsp = ws.data_ptr();
  }
  launch_skinny_gemm(c.data_ptr(), wsp, a.data_ptr(), w.data_ptr(), (int)M,
                     (int)N, (int)K, splits, gemm_stream());
  if (splits > 1)
    launch_reduce_splits(c.data_ptr(), wsp, splits, (long)(M * N),
                         gemm_stream());
  return c;
}
