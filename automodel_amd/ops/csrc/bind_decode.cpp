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

  m.def(
      "gemv_bf16(Tensor x, Tensor w, Tensor? bias, bool relu2=False, bool out_f32=False) "
      "-> Tensor");
  m.impl("gemv_bf16", &amd_ops::gemv_bf16);
  m.def("gemm_skinny_bf16(Tensor x, Tensor w, bool relu2, bool out_f32) -> Tensor");
  m.impl("gemm_skinny_bf16", &amd_ops::gemm_skinny_bf16);

  m.def("embed_rms_norm(Tensor ids, Tensor table, Tensor w, float eps) -> Tensor");
  m.impl("embed_rms_norm", &amd_ops::embed_rms_norm);
  m.def("residual_rms_norm(Tensor x, Tensor w, float eps) -> Tensor");
  m.impl("residual_rms_norm", &amd_ops::residual_rms_norm);
  m.def(
      "residual_add_norm(Tensor(a!) x, Tensor y, Tensor w_post, float mult, float eps_post, "
      "Tensor? w_next, float eps_next) -> Tensor");
  m.impl("residual_add_norm", &amd_ops::residual_add_norm);
  m.def("concat_cast(Tensor a, Tensor b, bool to_bf16) -> Tensor");
  m.impl("concat_cast", &amd_ops::concat_cast);
  m.def("relu2_(Tensor(a!) x) -> Tensor(a!)");
  m.impl("relu2_", &amd_ops::relu2_);

  m.def(
      "latent_prep(Tensor qkv, Tensor w, float eps, Tensor cos, Tensor sin, Tensor pos, "
      "Tensor? slot, Tensor(a!)? cache, int heads, int dn, int dr, int head_pad, int rows_pad) "
      "-> (Tensor, Tensor, Tensor)");
  m.impl("latent_prep", &amd_ops::latent_prep);
  m.def(
      "latent_assemble(Tensor kv, Tensor kr, int heads, int dn, int dv, int k_pad, int v_pad, "
      "int n_tok) -> (Tensor, Tensor)");
  m.impl("latent_assemble", &amd_ops::latent_assemble);
  m.def(
      "attn_rows(Tensor q, Tensor k, Tensor v, Tensor base, Tensor count, float scale, "
      "bool out_f32) -> Tensor");
  m.impl("attn_rows", &amd_ops::attn_rows);
  m.def(
      "latent_decode_prep(Tensor qkv, Tensor w_uk, Tensor w_norm, float eps, Tensor cos, "
      "Tensor sin, Tensor pos, Tensor slot, Tensor(a!) cache, int heads, int dn, int dr) "
      "-> Tensor");
  m.impl("latent_decode_prep", &amd_ops::latent_decode_prep);
  m.def(
      "latent_decode_attn(Tensor q, Tensor cache, Tensor slot, Tensor pos, int rank, int rot, "
      "float scale, int splits) -> (Tensor, Tensor)");
  m.impl("latent_decode_attn", &amd_ops::latent_decode_attn);
  m.def(
      "latent_decode_combine(Tensor part_o, Tensor? part_ml, Tensor w_uv, int dv) -> Tensor");
  m.impl("latent_decode_combine", &amd_ops::latent_decode_combine);
}
