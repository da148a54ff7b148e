// Declarations of all HIP op entry points (implemented in the sibling .hip TUs).
#pragma once

#include <ATen/ATen.h>
#include <tuple>

namespace amd_ops {

std::tuple<at::Tensor, at::Tensor> rms_norm_fwd(const at::Tensor& x, const at::Tensor& w,
                                                double eps);
std::tuple<at::Tensor, at::Tensor> rms_norm_bwd(const at::Tensor& dy, const at::Tensor& x,
                                                const at::Tensor& w, const at::Tensor& invrms);

std::tuple<at::Tensor, at::Tensor> rope_fwd(const at::Tensor& q, const at::Tensor& k,
                                            const at::Tensor& cosb, const at::Tensor& sinb,
                                            bool backward);

at::Tensor swiglu_fwd(const at::Tensor& g, const at::Tensor& u);
at::Tensor swiglu_cat_fwd(const at::Tensor& gu);
at::Tensor swiglu_cat_bwd(const at::Tensor& dy, const at::Tensor& gu);
std::tuple<at::Tensor, at::Tensor> swiglu_bwd(const at::Tensor& dy, const at::Tensor& g,
                                              const at::Tensor& u);

void adamw_step(at::Tensor param, at::Tensor grad, at::Tensor master, at::Tensor m,
                at::Tensor v, int64_t step, double lr, double beta1, double beta2,
                double eps, double weight_decay);

std::tuple<at::Tensor, at::Tensor> flash_attn_fwd(
    const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, double scale,
    bool causal, int64_t q_start,
    const std::optional<at::Tensor>& doc_start = std::nullopt,
    const std::optional<at::Tensor>& sink = std::nullopt);
std::tuple<at::Tensor, at::Tensor, at::Tensor> flash_attn_bwd(
    const at::Tensor& dout, const at::Tensor& q, const at::Tensor& k, const at::Tensor& v,
    const at::Tensor& o, const at::Tensor& lse, double scale, bool causal,
    int64_t q_start,
    const std::optional<at::Tensor>& doc_start = std::nullopt,
    const std::optional<at::Tensor>& doc_end = std::nullopt);

at::Tensor mfma_probe(const at::Tensor& a, const at::Tensor& b);
at::Tensor tr16_probe(const at::Tensor& pattern);

std::tuple<at::Tensor, at::Tensor> ce_fwd_logits(const at::Tensor& logits,
                                                 const at::Tensor& labels,
                                                 at::Tensor loss_sum);
void ce_bwd_logits(at::Tensor logits, const at::Tensor& labels, const at::Tensor& lse,
                   const at::Tensor& dloss, int64_t vocab_offset);
std::tuple<at::Tensor, at::Tensor> ce_stats_logits(const at::Tensor& logits);

std::tuple<at::Tensor, at::Tensor> fused_ce_fwd(const at::Tensor& hidden,
                                                const at::Tensor& weight,
                                                const at::Tensor& labels);

std::tuple<at::Tensor, at::Tensor, at::Tensor> soft_ce_fwd(const at::Tensor& s,
                                                           const at::Tensor& t);
at::Tensor soft_ce_bwd(const at::Tensor& s, const at::Tensor& t,
                       const at::Tensor& lse_s, const at::Tensor& lse_t,
                       const at::Tensor& dloss);

at::Tensor nf4_dequant(const at::Tensor& packed, const at::Tensor& absmax,
                       int64_t block_size, int64_t rows, int64_t cols);
at::Tensor fp8_cast(const at::Tensor& x, const at::Tensor& scale, at::Tensor amax_out,
                    bool e5m2);
at::Tensor fp8_transpose(const at::Tensor& x8);
at::Tensor lora_fused_fwd(const at::Tensor& x, const at::Tensor& A,
                          const at::Tensor& B, double scale);
at::Tensor sgmv_fused_fwd(const at::Tensor& x, const at::Tensor& A,
                          const at::Tensor& B, const at::Tensor& scales,
                          const at::Tensor& offs, const at::Tensor& tile_map,
                          const std::optional<at::Tensor>& n_tiles = std::nullopt);

at::Tensor gemv_bf16(const at::Tensor& x, const at::Tensor& w,
                     const c10::optional<at::Tensor>& bias, bool relu2 = false,
                     bool out_f32 = false, int64_t group_n = 0);
at::Tensor gemm_skinny_bf16(const at::Tensor& x, const at::Tensor& w, bool relu2, bool out_f32,
                            int64_t group_n = 0);

std::tuple<at::Tensor, at::Tensor, at::Tensor> build_group_plan(
    const at::Tensor& counts, int64_t M, int64_t bm = 128);
at::Tensor grouped_gemm_nt(const at::Tensor& x, const at::Tensor& w,
                           const at::Tensor& offs, const at::Tensor& tile_map,
                           const std::optional<at::Tensor>& n_tiles = std::nullopt,
                           int64_t bm = 128);
at::Tensor grouped_gemm_nn(const at::Tensor& g, const at::Tensor& w,
                           const at::Tensor& offs, const at::Tensor& tile_map,
                           const std::optional<at::Tensor>& n_tiles = std::nullopt);
at::Tensor grouped_gemm_tn(const at::Tensor& g, const at::Tensor& x,
                           const at::Tensor& offs, int64_t E);
at::Tensor grouped_gemm_nt_fp8(const at::Tensor& x8, const at::Tensor& w8,
                               const at::Tensor& offs, const at::Tensor& tile_map,
                               const at::Tensor& scale,
                               const std::optional<at::Tensor>& n_tiles = std::nullopt,
                               int64_t bm = 128);
at::Tensor transpose_bf16(const at::Tensor& in);
at::Tensor permute_gather(const at::Tensor& x, const at::Tensor& src);
at::Tensor unpermute_combine(const at::Tensor& yp, const at::Tensor& pos,
                             const at::Tensor& probs);

// --- inference: f32 residual stream (residual_norm.hip) ---
at::Tensor embed_rms_norm(const at::Tensor& ids, const at::Tensor& table, const at::Tensor& w,
                          double eps);
at::Tensor residual_rms_norm(const at::Tensor& x, const at::Tensor& w, double eps);
at::Tensor residual_add_norm(at::Tensor x, const at::Tensor& y, const at::Tensor& w_post,
                             double mult, double eps_post,
                             const std::optional<at::Tensor>& w_next, double eps_next);
at::Tensor concat_cast(const at::Tensor& a, const at::Tensor& b, bool to_bf16);
at::Tensor relu2_(at::Tensor x);

// --- inference: latent attention (latent_attn.hip, latent_decode.hip) ---
std::tuple<at::Tensor, at::Tensor, at::Tensor> latent_prep(
    const at::Tensor& qkv, const at::Tensor& w, double eps, const at::Tensor& cos,
    const at::Tensor& sin, const at::Tensor& pos, const std::optional<at::Tensor>& slot,
    const std::optional<at::Tensor>& cache, int64_t heads, int64_t dn, int64_t dr,
    int64_t head_pad, int64_t rows_pad);
std::tuple<at::Tensor, at::Tensor> latent_assemble(const at::Tensor& kv, const at::Tensor& kr,
                                                   int64_t heads, int64_t dn, int64_t dv,
                                                   int64_t k_pad, int64_t v_pad, int64_t n_tok);
at::Tensor attn_rows(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v,
                     const at::Tensor& base, const at::Tensor& count, double scale, bool out_f32,
                     const std::optional<at::Tensor>& sink = std::nullopt);
at::Tensor latent_decode_prep(const at::Tensor& qkv, const at::Tensor& w_uk,
                              const at::Tensor& w_norm, double eps, const at::Tensor& cos,
                              const at::Tensor& sin, const at::Tensor& pos, const at::Tensor& slot,
                              at::Tensor cache, int64_t heads, int64_t dn, int64_t dr);
std::tuple<at::Tensor, at::Tensor> latent_decode_attn(const at::Tensor& q, const at::Tensor& cache,
                                                      const at::Tensor& slot, const at::Tensor& pos,
                                                      int64_t rank, int64_t rot, double scale,
                                                      int64_t splits);
at::Tensor latent_decode_combine(const at::Tensor& part_o,
                                 const std::optional<at::Tensor>& part_ml, const at::Tensor& w_uv,
                                 int64_t dv);

// --- inference: grouped attention, chunks, sinks (gqa_attn.hip) ---
std::tuple<at::Tensor, at::Tensor, at::Tensor> gqa_prep(
    const at::Tensor& proj, const at::Tensor& cos, const at::Tensor& sin, const at::Tensor& pos,
    const std::optional<at::Tensor>& slot, const std::optional<at::Tensor>& seq_end,
    const std::optional<at::Tensor>& cu_seqlens, const std::optional<at::Tensor>& k_cache,
    const std::optional<at::Tensor>& v_cache, int64_t chunk, int64_t heads, int64_t kv_heads,
    int64_t d, int64_t dv, int64_t head_pad, int64_t v_pad, int64_t rows_pad, bool decode);
at::Tensor gqa_decode_attn(const at::Tensor& q, const at::Tensor& k_cache,
                           const at::Tensor& v_cache, const at::Tensor& slot,
                           const at::Tensor& pos, const std::optional<at::Tensor>& sink,
                           int64_t chunk, int64_t dv, double scale, int64_t splits);

// --- inference: hyper-connections (hyper.hip) ---
std::tuple<at::Tensor, at::Tensor> hyper_embed(const at::Tensor& ids, const at::Tensor& table,
                                               double scale, const at::Tensor& w_in,
                                               const at::Tensor& w_norm, double eps);
at::Tensor hyper_step(at::Tensor x, const at::Tensor& y, const std::optional<at::Tensor>& y2,
                      const std::optional<at::Tensor>& w_y, const std::optional<at::Tensor>& w_y2,
                      const at::Tensor& w_mix, const at::Tensor& w_out,
                      const std::optional<at::Tensor>& w_in, const at::Tensor& w_norm, double eps,
                      bool keep);
at::Tensor clamped_glu(const at::Tensor& gu, double limit, double alpha);

// --- inference: linear recurrences (linear_scan.hip) ---
at::Tensor causal_conv_silu(const at::Tensor& x, const at::Tensor& w, const at::Tensor& bias,
                            const at::Tensor& pos, const std::optional<at::Tensor>& slot,
                            const std::optional<at::Tensor>& seq_end,
                            const std::optional<at::Tensor>& state);
at::Tensor token_shift(const at::Tensor& h, const at::Tensor& mu, const at::Tensor& pos,
                       const std::optional<at::Tensor>& slot,
                       const std::optional<at::Tensor>& seq_end,
                       const std::optional<at::Tensor>& state);
at::Tensor gated_group_norm(const at::Tensor& y, const at::Tensor& z, const at::Tensor& w,
                            int64_t groups, double eps, bool gate_first);
at::Tensor ssd_prompt(const at::Tensor& xbc, const at::Tensor& dt_in, const at::Tensor& dt_bias,
                      const at::Tensor& a_log, const at::Tensor& d_skip, const at::Tensor& cu,
                      const std::optional<at::Tensor>& slot,
                      const std::optional<at::Tensor>& state, int64_t groups, int64_t N,
                      int64_t max_len);
at::Tensor ssd_decode(const at::Tensor& xbc, const at::Tensor& dt_in, const at::Tensor& dt_bias,
                      const at::Tensor& a_log, const at::Tensor& d_skip, const at::Tensor& slot,
                      at::Tensor state, int64_t groups, int64_t N);
at::Tensor wkv_prompt(const at::Tensor& r, const at::Tensor& k, const at::Tensor& v,
                      at::Tensor low, const at::Tensor& w0, const at::Tensor& u,
                      const at::Tensor& cu, const std::optional<at::Tensor>& slot,
                      const std::optional<at::Tensor>& state, int64_t max_len);
at::Tensor wkv_decode(const at::Tensor& proj, const at::Tensor& w2, const at::Tensor& w0,
                      const at::Tensor& u, const at::Tensor& w_norm, double eps,
                      const at::Tensor& slot, at::Tensor state);

}  // namespace amd_ops
