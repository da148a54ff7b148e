// Registration of the inference ops (attention forward, latent attention,
// residual norms, decode GEMV) as a fragment of the amd_ops namespace: part of
// libamd_ops.so, and of the small libamd_ops_decode.so (ops/build.py --decode).

#include <torch/library.h>

#include "ops_api.h"

TORCH_LIBRARY_FRAGMENT(amd_ops, m) {
  m.def(
      "flash_attn_fwd(Tensor q, Tensor k, Tensor v, float scale, bool causal, "
      "int q_start=0, Tensor? doc_start=None) -> (Tensor, Tensor)");
  m.impl("flash_attn_fwd", &amd_ops::flash_attn_fwd);

  m.def("gemv_bf16(Tensor x, Tensor w, Tensor? bias) -> Tensor");
  m.impl("gemv_bf16", &amd_ops::gemv_bf16);
}
