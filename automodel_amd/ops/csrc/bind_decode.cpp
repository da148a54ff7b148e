// Registration of the inference ops (attention forward, latent and grouped
// attention, linear recurrences, residual norms, hyper-connections, decode GEMV) as a fragment of the amd_ops namespace: part of
// libamd_ops.so, and of the small libamd_ops_decode.so (ops/build.py --decode).

#include <torch/library.h>

#include "ops_api.h"

TORCH_LIBRARY_FRAGMENT(amd_ops, m) {
  m.def(
      "flash_attn_fwd(Tensor q, Tensor k, Tensor v, float scale, bool causal, "
      "int q_start=0, Tensor? doc_start=None, Tensor? sink=None) -> (Tensor, Tensor)");
  m.impl("flash_attn_fwd", &amd_ops::flash_attn_fwd);

  m.def(
      "gemv_bf16(Tensor x, Tensor w, Tensor? bias, bool relu2=False, bool out_f32=False, "
      "int group_n=0) -> Tensor");
  m.impl("gemv_bf16", &amd_ops::gemv_bf16);
  m.def(
      "gemm_skinny_bf16(Tensor x, Tensor w, bool relu2, bool out_f32, int group_n=0) -> Tensor");
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
      "bool out_f32, Tensor? sink=None) -> Tensor");
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

  m.def(
      "gqa_prep(Tensor proj, Tensor cos, Tensor sin, Tensor pos, Tensor? slot, Tensor? seq_end, "
      "Tensor? cu_seqlens, Tensor(a!)? k_cache, Tensor(b!)? v_cache, int chunk, int heads, "
      "int kv_heads, int d, int dv, int head_pad, int v_pad, int rows_pad, bool decode) "
      "-> (Tensor, Tensor, Tensor)");
  m.impl("gqa_prep", &amd_ops::gqa_prep);
  m.def(
      "gqa_decode_attn(Tensor q, Tensor k_cache, Tensor v_cache, Tensor slot, Tensor pos, "
      "Tensor? sink, int chunk, int dv, float scale, int splits) -> Tensor");
  m.impl("gqa_decode_attn", &amd_ops::gqa_decode_attn);

  m.def(
      "hyper_embed(Tensor ids, Tensor table, float scale, Tensor w_in, Tensor w_norm, float eps) "
      "-> (Tensor, Tensor)");
  m.impl("hyper_embed", &amd_ops::hyper_embed);
  m.def(
      "hyper_step(Tensor(a!) x, Tensor y, Tensor? y2, Tensor? w_y, Tensor? w_y2, Tensor w_mix, "
      "Tensor w_out, Tensor? w_in, Tensor w_norm, float eps, bool keep) -> Tensor");
  m.impl("hyper_step", &amd_ops::hyper_step);
  m.def("clamped_glu(Tensor gu, float limit, float alpha) -> Tensor");
  m.impl("clamped_glu", &amd_ops::clamped_glu);

  m.def(
      "causal_conv_silu(Tensor x, Tensor w, Tensor bias, Tensor pos, Tensor? slot, "
      "Tensor? seq_end, Tensor(a!)? state) -> Tensor");
  m.impl("causal_conv_silu", &amd_ops::causal_conv_silu);
  m.def(
      "token_shift(Tensor h, Tensor mu, Tensor pos, Tensor? slot, Tensor? seq_end, "
      "Tensor(a!)? state) -> Tensor");
  m.impl("token_shift", &amd_ops::token_shift);
  m.def(
      "gated_group_norm(Tensor y, Tensor z, Tensor w, int groups, float eps, bool gate_first) "
      "-> Tensor");
  m.impl("gated_group_norm", &amd_ops::gated_group_norm);
  m.def(
      "ssd_prompt(Tensor xbc, Tensor dt, Tensor dt_bias, Tensor a_log, Tensor d_skip, "
      "Tensor cu_seqlens, Tensor? slot, Tensor(a!)? state, int groups, int n, int max_len) "
      "-> Tensor");
  m.impl("ssd_prompt", &amd_ops::ssd_prompt);
  m.def(
      "ssd_decode(Tensor xbc, Tensor dt, Tensor dt_bias, Tensor a_log, Tensor d_skip, "
      "Tensor slot, Tensor(a!) state, int groups, int n) -> Tensor");
  m.impl("ssd_decode", &amd_ops::ssd_decode);
  m.def(
      "wkv_prompt(Tensor r, Tensor k, Tensor v, Tensor(a!) low, Tensor w0, Tensor u, "
      "Tensor cu_seqlens, Tensor? slot, Tensor(b!)? state, int max_len) -> Tensor");
  m.impl("wkv_prompt", &amd_ops::wkv_prompt);
  m.def(
      "wkv_decode(Tensor proj, Tensor w2, Tensor w0, Tensor u, Tensor w_norm, float eps, "
      "Tensor slot, Tensor(a!) state) -> Tensor");
  m.impl("wkv_decode", &amd_ops::wkv_decode);
}
