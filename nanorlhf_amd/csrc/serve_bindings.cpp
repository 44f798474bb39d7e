// Python bindings of the serving kernels: paged cache, attention over it,
// linear attention with its state slots, residual-stream operations.
#include <torch/extension.h>

using OptTensor = c10::optional<torch::Tensor>;

// kvcache.hip
void kv_append(torch::Tensor k, torch::Tensor v, torch::Tensor slots,
               torch::Tensor k_cache, torch::Tensor v_cache);
torch::Tensor paged_attn_decode(torch::Tensor q, torch::Tensor k_cache,
                                torch::Tensor v_cache, torch::Tensor block_tables,
                                torch::Tensor seq_lens, double scale);
void paged_attn_decode_window(torch::Tensor q, torch::Tensor k_cache, torch::Tensor v_cache,
                              torch::Tensor block_tables, torch::Tensor seq_lens,
                              torch::Tensor out, double scale, long size, long keep,
                              OptTensor uncs);
// paged_attention.hip
void paged_attn_varlen(torch::Tensor q, torch::Tensor kc, torch::Tensor vc, torch::Tensor cu,
                       torch::Tensor seq_lens, torch::Tensor bt, torch::Tensor out, long max_q,
                       double scale, long size, long keep, OptTensor uncs);
void paged_attn_plain(torch::Tensor q, torch::Tensor kc, torch::Tensor vc, torch::Tensor row_seq,
                      torch::Tensor positions, torch::Tensor bt, torch::Tensor out, double scale,
                      long size, long keep, OptTensor uncs);
// linear_attn.hip
void linear_attn_chunked(torch::Tensor q, torch::Tensor k, torch::Tensor v, torch::Tensor pw,
                         OptTensor cs, bool interleaved, bool silu, double kscale,
                         torch::Tensor chunks, torch::Tensor first, torch::Tensor slots,
                         torch::Tensor fresh, torch::Tensor state, OptTensor gate, double eps,
                         torch::Tensor o);
void linear_attn_decode(torch::Tensor q, torch::Tensor k, torch::Tensor v, torch::Tensor pw,
                        OptTensor cs, bool interleaved, bool silu, double kscale,
                        torch::Tensor slots, torch::Tensor seq_lens, torch::Tensor state,
                        OptTensor gate, double eps, torch::Tensor o);
// stream.hip
torch::Tensor residual_group_norm(torch::Tensor x, OptTensor delta, OptTensor embed,
                                  OptTensor ids, torch::Tensor w, long groups, double mult,
                                  double eps);
void gated_norm(torch::Tensor in, OptTensor w, torch::Tensor gate, torch::Tensor out,
                long groups, long act, double eps);
void gelu_glu(torch::Tensor gate, torch::Tensor up, torch::Tensor out, long pad, long tail);
torch::Tensor rope_angles(torch::Tensor positions, torch::Tensor freqs);
torch::Tensor rotary_qkv(torch::Tensor proj, long qoff, long koff, long voff, OptTensor qw,
                         OptTensor kw, OptTensor csk, OptTensor csv, torch::Tensor slots,
                         torch::Tensor kc, torch::Tensor vc, long H, long G, long D, long V,
                         bool interleaved, double eps);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("kv_append", &kv_append);
  m.def("paged_attn_decode", &paged_attn_decode);
  m.def("paged_attn_decode_window", &paged_attn_decode_window);
  m.def("paged_attn_varlen", &paged_attn_varlen);
  m.def("paged_attn_plain", &paged_attn_plain);
  m.def("linear_attn_chunked", &linear_attn_chunked);
  m.def("linear_attn_decode", &linear_attn_decode);
  m.def("residual_group_norm", &residual_group_norm);
  m.def("gated_norm", &gated_norm);
  m.def("gelu_glu", &gelu_glu);
  m.def("rope_angles", &rope_angles);
  m.def("rotary_qkv", &rotary_qkv);
}
