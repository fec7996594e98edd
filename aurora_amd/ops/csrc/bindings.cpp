// Python bindings of the decoder kernels (gfx950).
#include <torch/extension.h>

torch::Tensor rmsnorm(torch::Tensor x, torch::Tensor weight, double eps);
std::vector<torch::Tensor> rmsnorm_residual(torch::Tensor x, torch::Tensor res,
                                            torch::Tensor weight, double eps);
torch::Tensor silu_mul(torch::Tensor gu);
void rope_apply_(torch::Tensor q, torch::Tensor k, torch::Tensor positions,
                 torch::Tensor cos_sin);
void kv_cache_write(torch::Tensor k, torch::Tensor v, torch::Tensor kc,
                    torch::Tensor vc, torch::Tensor slots);
torch::Tensor paged_attention_decode(torch::Tensor q, torch::Tensor kc,
                                     torch::Tensor vc, torch::Tensor bt,
                                     torch::Tensor ctx, double scale);
torch::Tensor attention_prefill_paged(torch::Tensor q, torch::Tensor kc,
                                      torch::Tensor vc, torch::Tensor bt,
                                      torch::Tensor cu_q, torch::Tensor ctx,
                                      double scale);
torch::Tensor skinny_gemm(torch::Tensor x, torch::Tensor w);
torch::Tensor fused_rope_kv_write(torch::Tensor qkv, torch::Tensor positions,
                                  torch::Tensor slots, torch::Tensor cos_sin,
                                  torch::Tensor kc, torch::Tensor vc,
                                  long Hq, long Hkv);
torch::Tensor skinny_gemm_ex(torch::Tensor x, torch::Tensor w, long s_target, long unroll);
torch::Tensor skinny_gemm2_ex(torch::Tensor x, torch::Tensor w, long s_target);
torch::Tensor skinny_gemm3_ex(torch::Tensor x, torch::Tensor w, long s_target);
torch::Tensor moe_grouped_gemm(torch::Tensor xp, torch::Tensor w,
                               torch::Tensor starts, torch::Tensor counts);
// ---- layer-listed decoders
using OptT = c10::optional<torch::Tensor>;
std::vector<torch::Tensor> residual_rmsnorm(torch::Tensor x, torch::Tensor weight, OptT delta,
                                            OptT gate_pre, OptT gate_bias, OptT y, OptT place,
                                            OptT gate, OptT post, OptT step, OptT conv_w, OptT ring,
                                            OptT pos, OptT slots, double eps, double offset,
                                            bool to_bf16);
void embed_pairs(torch::Tensor ids, torch::Tensor table, double scale, torch::Tensor pairs,
                 long mul_prev, long mul_cur, torch::Tensor weight, double eps,
                 torch::Tensor prev, OptT cu, torch::Tensor starts, torch::Tensor slots,
                 torch::Tensor out);
long short_conv_rows();
void short_conv_add(torch::Tensor h, torch::Tensor w, torch::Tensor ring, OptT cu, OptT bseq,
                    OptT boff, torch::Tensor starts, torch::Tensor slots, torch::Tensor out);
torch::Tensor xielu(torch::Tensor z, torch::Tensor act);
void latent_front(torch::Tensor proj, long c0, long rank, OptT weight, double eps, long k0,
                  long key_at, OptT cos_sin, OptT pos, torch::Tensor slots,
                  torch::Tensor cache, long q0, OptT q_weight, OptT cq);
torch::Tensor gather_latents(torch::Tensor cache, torch::Tensor rows);
void rotate_heads(torch::Tensor x, torch::Tensor pos, torch::Tensor cos_sin,
                  torch::Tensor out);
void head_linear(torch::Tensor x, torch::Tensor w, OptT gate, torch::Tensor out, OptT turn_x,
                 OptT turn_pos, OptT turn_cs, OptT turn_out);
torch::Tensor latent_attention(torch::Tensor q, torch::Tensor cache, torch::Tensor bt, OptT cu,
                               torch::Tensor ctx, OptT bseq, OptT boff, long rows,
                               double scale, OptT sink, long VR, long window);
void latent_attention_rows(torch::Tensor q, torch::Tensor cache, torch::Tensor bt, OptT cu,
                           torch::Tensor ctx, OptT row_seq, OptT row_off, double scale,
                           OptT sink, long window, torch::Tensor out);
void tailed_attention_prefill(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                              torch::Tensor tail, torch::Tensor bt, torch::Tensor cu_q,
                              torch::Tensor ctx, torch::Tensor bseq, torch::Tensor boff,
                              double scale, long window, torch::Tensor out);
long conv_qkv_rows();
void conv_qkv(torch::Tensor proj, long q0, long k0, long v0, torch::Tensor w,
              torch::Tensor turn, OptT value_turn, torch::Tensor ring, torch::Tensor kv_slots,
              OptT cu, OptT bseq, OptT boff, torch::Tensor starts, torch::Tensor slots,
              torch::Tensor kc, torch::Tensor vc, torch::Tensor q, long d, long dv);
void sink_attention_prefill(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                            torch::Tensor bt, torch::Tensor cu_q, torch::Tensor ctx,
                            torch::Tensor bseq, torch::Tensor boff, double scale,
                            torch::Tensor sink, torch::Tensor gate, torch::Tensor out);
torch::Tensor bias_kv_write(torch::Tensor proj, long q0, long k0, long v0,
                            torch::Tensor bias, torch::Tensor slots, torch::Tensor kc,
                            torch::Tensor vc, long Hq, long Hkv, long d, long dv);
long biased_prefill_rows(long G);
void biased_attention_prefill(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                              torch::Tensor bt, torch::Tensor cu_q, torch::Tensor ctx,
                              torch::Tensor bseq, torch::Tensor boff, double scale,
                              long window, long chunk, OptT slopes, OptT rates, OptT sink,
                              OptT turn, OptT gate, torch::Tensor out, long col, long dv,
                              double oscale);
void biased_attention_decode(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                             torch::Tensor bt, torch::Tensor ctx, double scale, long window,
                             long chunk, OptT slopes, OptT rates, OptT sink, OptT turn,
                             OptT gate, torch::Tensor out, long col, long dv, double oscale);
void biased_attention_rows(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                           torch::Tensor bt, OptT cu, torch::Tensor ctx, OptT row_seq,
                           OptT row_off, double scale, long window, long chunk, OptT slopes,
                           OptT rates, OptT sink, OptT turn, OptT gate, torch::Tensor out,
                           long col, long dv, double oscale);
void delta_prefill(torch::Tensor proj, torch::Tensor z, torch::Tensor conv_w,
                   torch::Tensor a_log, torch::Tensor dt_bias, torch::Tensor norm, long H,
                   long G, long d, long e, long taps, long q0, long k0, long v0, long b0,
                   double eps, torch::Tensor state, torch::Tensor ring, torch::Tensor cu,
                   torch::Tensor cseq, torch::Tensor coff, torch::Tensor cfirst,
                   torch::Tensor starts, torch::Tensor slots, torch::Tensor out, long col,
                   double oscale);
void delta_decode(torch::Tensor proj, torch::Tensor z, torch::Tensor conv_w,
                  torch::Tensor a_log, torch::Tensor dt_bias, torch::Tensor norm, long H,
                  long G, long d, long e, long taps, long q0, long k0, long v0, long b0,
                  double eps, torch::Tensor state, torch::Tensor ring, torch::Tensor starts,
                  torch::Tensor slots, torch::Tensor out, long col, double oscale);
void retention_prefill(torch::Tensor proj, torch::Tensor decay, torch::Tensor cos_sin,
                       long H, long d, long e, long rot, long q0, long k0, long v0, long g0,
                       double eps, torch::Tensor state, torch::Tensor cu, torch::Tensor cseq,
                       torch::Tensor coff, torch::Tensor cfirst, torch::Tensor starts,
                       torch::Tensor slots, torch::Tensor out);
void retention_decode(torch::Tensor proj, torch::Tensor decay, torch::Tensor cos_sin, long H,
                      long d, long e, long rot, long q0, long k0, long v0, long g0,
                      double eps, torch::Tensor state, torch::Tensor starts,
                      torch::Tensor slots, torch::Tensor out);
std::vector<torch::Tensor> moe_route(torch::Tensor h, torch::Tensor router,
                                     torch::Tensor bias, long top);
std::vector<torch::Tensor> moe_clamped_glu(torch::Tensor h, torch::Tensor sel,
                                           torch::Tensor w_gu, torch::Tensor w_dn,
                                           double limit, double alpha, double shift);
std::vector<torch::Tensor> moe_route_grouped(torch::Tensor h, torch::Tensor router,
                                             OptT correction, long top, long groups,
                                             long keep, double scale);
std::vector<torch::Tensor> moe_relu2(torch::Tensor h, torch::Tensor sel, torch::Tensor w_up,
                                     torch::Tensor w_dn);
torch::Tensor gelu(torch::Tensor z);
torch::Tensor relu2(torch::Tensor z);
torch::Tensor silu_glu(torch::Tensor z, long F);
torch::Tensor output_norm(torch::Tensor src, torch::Tensor x, torch::Tensor weight,
                          torch::Tensor bias, OptT delta, OptT gate, OptT y, OptT place,
                          OptT share, OptT kept, OptT coefs, OptT fw, OptT fb, double eps,
                          bool to_bf16);
torch::Tensor normed_qkv(torch::Tensor proj, long q0, long k0, long v0, torch::Tensor qw,
                         torch::Tensor kw, bool whole, double eps, OptT cos_sin, double coef,
                         long every, torch::Tensor pos, torch::Tensor slots, torch::Tensor kc,
                         torch::Tensor vc, long Hq, long Hkv, long d, long dv);
void head_delta_prefill(torch::Tensor proj, torch::Tensor conv_w, torch::Tensor a_log,
                        torch::Tensor dt_bias, torch::Tensor norm, long H, long G, long d,
                        long e, long taps, long q0, long k0, long v0, long b0, long a0,
                        long g0, double eps, torch::Tensor state, torch::Tensor ring,
                        torch::Tensor cu, torch::Tensor cseq, torch::Tensor coff,
                        torch::Tensor cfirst, torch::Tensor starts, torch::Tensor slots,
                        torch::Tensor out, long col, double oscale);
void head_delta_decode(torch::Tensor proj, torch::Tensor conv_w, torch::Tensor a_log,
                       torch::Tensor dt_bias, torch::Tensor norm, long H, long G, long d,
                       long e, long taps, long q0, long k0, long v0, long b0, long a0,
                       long g0, double eps, torch::Tensor state, torch::Tensor ring,
                       torch::Tensor starts, torch::Tensor slots, torch::Tensor out,
                       long col, double oscale);
void memory_prefill(torch::Tensor proj, torch::Tensor i_bias, torch::Tensor f_bias,
                    torch::Tensor norm, long H, long d, long e, long q0, long k0, long v0,
                    long i0, long f0, long g0, double cap, double eps, torch::Tensor state,
                    torch::Tensor nstate, torch::Tensor mstate, torch::Tensor cu,
                    torch::Tensor cseq, torch::Tensor coff, torch::Tensor cfirst,
                    torch::Tensor starts, torch::Tensor slots, torch::Tensor out, long col,
                    double oscale);
void memory_decode(torch::Tensor proj, torch::Tensor i_bias, torch::Tensor f_bias,
                   torch::Tensor norm, long H, long d, long e, long q0, long k0, long v0,
                   long i0, long f0, long g0, double cap, double eps, torch::Tensor state,
                   torch::Tensor nstate, torch::Tensor mstate, torch::Tensor starts,
                   torch::Tensor slots, torch::Tensor out, long col, double oscale);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("rmsnorm", &rmsnorm, "fused RMSNorm (bf16, gfx950)");
  m.def("rmsnorm_residual", &rmsnorm_residual, "fused residual-add + RMSNorm");
  m.def("silu_mul", &silu_mul, "fused SiLU(gate)*up");
  m.def("rope_apply_", &rope_apply_, "in-place RoPE on q/k");
  m.def("kv_cache_write", &kv_cache_write, "scatter K/V into paged cache");
  m.def("paged_attention_decode", &paged_attention_decode, "paged GQA decode attention");
  m.def("attention_prefill_paged", &attention_prefill_paged,
        "MFMA flash prefill over paged KV");
  m.def("skinny_gemm", &skinny_gemm, "decode-path skinny GEMM (M<=64)");
  m.def("fused_rope_kv_write", &fused_rope_kv_write,
        "fused qkv split + RoPE + paged KV scatter");
  m.def("skinny_gemm_ex", &skinny_gemm_ex, "skinny GEMM with tuning knobs");
  m.def("skinny_gemm2_ex", &skinny_gemm2_ex, "LDS-staged skinny GEMM (M<=64)");
  m.def("skinny_gemm3_ex", &skinny_gemm3_ex, "glds double-buffered projection GEMM (M<=256)");
  m.def("moe_grouped_gemm", &moe_grouped_gemm,
        "packed per-expert grouped GEMM (skips unrouted experts)");
  m.def("residual_rmsnorm", &residual_rmsnorm,
        "fp32 residual add (dense, gated or routed rows, normed or not, pass vector) + RMSNorm, "
        "+ input convolution of single tokens");
  m.def("embed_pairs", &embed_pairs, "token + token-pair embedding, normed");
  m.def("short_conv_rows", &short_conv_rows);
  m.def("short_conv_add", &short_conv_add, "input plus its causal convolution");
  m.def("xielu", &xielu, "xIELU activation");
  m.def("latent_front", &latent_front,
        "latent norm + rotated key part + paged scatter, norm of the queries' latent");
  m.def("gather_latents", &gather_latents, "cached latent rows, packed");
  m.def("rotate_heads", &rotate_heads, "rotary positions of neighbouring pairs");
  m.def("head_linear", &head_linear,
        "per-head product with an optional gate, or beside rotated dimensions");
  m.def("latent_attention", &latent_attention,
        "MFMA attention in the latents' space over the paged cache, with sink and window");
  m.def("latent_attention_rows", &latent_attention_rows,
        "any latent width / float32 latent attention with sink and window");
  m.def("sink_attention_prefill", &sink_attention_prefill,
        "MFMA flash prefill with a sink and a gate per head");
  m.def("tailed_attention_prefill", &tailed_attention_prefill,
        "MFMA flash prefill whose heads share their keys' last dimensions, with a window");
  m.def("conv_qkv_rows", &conv_qkv_rows);
  m.def("conv_qkv", &conv_qkv,
        "causal convolution + rotation of heads and values + paged KV scatter");
  m.def("bias_kv_write", &bias_kv_write, "bias + head split + paged KV scatter");
  m.def("biased_prefill_rows", &biased_prefill_rows);
  m.def("biased_attention_prefill", &biased_attention_prefill,
        "MFMA flash prefill with distance bias, window or chunks, sink, turn and gate");
  m.def("biased_attention_decode", &biased_attention_decode,
        "paged decode with distance bias, window or chunks, sink, turn and gate");
  m.def("biased_attention_rows", &biased_attention_rows,
        "any head width / float32 attention with distance bias, window or chunks, sink, "
        "turn and gate");
  m.def("delta_prefill", &delta_prefill, "gated delta rule, chunked");
  m.def("delta_decode", &delta_decode, "gated delta rule, one token per sequence");
  m.def("retention_prefill", &retention_prefill, "retention, chunked");
  m.def("retention_decode", &retention_decode, "retention, one token per sequence");
  m.def("moe_route", &moe_route, "fp32 router, top choice, softmax over the chosen");
  m.def("moe_route_grouped", &moe_route_grouped,
        "fp32 sigmoid or softmax router, top choice among the best groups");
  m.def("moe_relu2", &moe_relu2, "sorted grouped squared-relu experts");
  m.def("moe_clamped_glu", &moe_clamped_glu, "sorted grouped clamped-GLU experts");
  m.def("head_delta_prefill", &head_delta_prefill,
        "gated delta rule with a decay per head, chunked");
  m.def("head_delta_decode", &head_delta_decode,
        "gated delta rule with a decay per head, one token per sequence");
  m.def("memory_prefill", &memory_prefill, "matrix memory (mLSTM), chunked");
  m.def("memory_decode", &memory_decode, "matrix memory (mLSTM), one token per sequence");
  m.def("output_norm", &output_norm,
        "sub-layer result put together, layer norm, fp32 residual, depth average, "
        "final norm");
  m.def("normed_qkv", &normed_qkv,
        "head norms + rotation + temperature + paged KV scatter");
  m.def("gelu", &gelu, "exact gelu");
  m.def("relu2", &relu2, "squared relu");
  m.def("silu_glu", &silu_glu, "silu(gate) * up");
}
