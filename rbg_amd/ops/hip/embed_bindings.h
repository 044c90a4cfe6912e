// Binding of the scaled embedding, for every extension that links embed.hip.
#pragma once
#include "bind_util.h"

extern "C" void launch_embed_stream(float*, const void*, const long*, float,
                                    int, int, int, int, hipStream_t);

// f32 [tokens, copies * width]
[[maybe_unused]] static torch::Tensor embed_stream(torch::Tensor tokens,
                                                   torch::Tensor table,
                                                   double scale,
                                                   int64_t copies) {
  check_rows(table, "table");
  TORCH_CHECK(table.is_contiguous() && tokens.is_cuda() &&
              tokens.scalar_type() == torch::kInt64 && tokens.is_contiguous(),
              "tokens must be int64 on GPU, table contiguous");
  TORCH_CHECK(copies > 0, "copies");
  auto x = torch::empty({tokens.numel(), copies * table.size(1)},
                        table.options().dtype(torch::kFloat32));
  if (tokens.numel())
    launch_embed_stream(x.data_ptr<float>(), table.data_ptr(),
                        (const long*)tokens.data_ptr<int64_t>(), (float)scale,
                        (int)tokens.numel(), (int)table.size(1), (int)copies,
                        is_f32(table), current_stream());
  return x;
}
