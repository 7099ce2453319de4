// pybind11 module `_native`: kernel launchers (raw device pointers + stream handles passed as
// integers from the python ops layer, which owns shape/dtype validation) and the native host
// runtime (tokenizer, paged-KV block manager, retrieval post-processing).
#include <hip/hip_runtime.h>
#include <pybind11/numpy.h>
#include <pybind11/pybind11.h>
#include <pybind11/stl.h>

#include <stdexcept>
#include <string>

#include "kernels/launchers.h"
#include "runtime/json_grammar.h"
#include "runtime/kv_manager.h"
#include "runtime/rag.h"
#include "runtime/tokenizer.h"
#include "runtime/trace.h"

namespace py = pybind11;
using u = uintptr_t;

#define VP(x) reinterpret_cast<void*>(x)
#define CVP(x) reinterpret_cast<const void*>(x)
#define ST(x) reinterpret_cast<hipStream_t>(x)

static void check(int err, const char* name) {
  if (err) throw std::runtime_error(std::string("dab kernel '") + name + "' failed: " + hipGetErrorString((hipError_t)err));
}

PYBIND11_MODULE(_native, m) {
  m.doc() = "MI355X (gfx950) kernels and native runtime of django_assistant_bot_amd";
  m.def("roctx_available", &dab::trace::available);
  // one-shot all-reduce over IPC peer buffers (parallel/custom_allreduce.py)
  m.def("allreduce_signal_bytes", &dab::allreduce_signal_bytes);
  m.def("custom_allreduce", [](const std::vector<uintptr_t>& bases, int rank, u data, long nbytes, long half_bytes,
                               long spin_limit, u s) {
    check(dab::custom_allreduce(bases, rank, VP(data), nbytes, half_bytes, spin_limit, ST(s)), "custom_allreduce");
  });
  m.def("custom_allreduce_rmsnorm", [](const std::vector<uintptr_t>& bases, int rank, u slabs, int S, long slab_stride,
                                       u x, u res_in, u res_out, u out, u w, int rows, int cols, float eps,
                                       long half_bytes, long spin_limit, u s) {
    check(dab::custom_allreduce_rmsnorm(bases, rank, (const float*)slabs, S, slab_stride, CVP(x), CVP(res_in),
                                        VP(res_out), VP(out), CVP(w), rows, cols, eps, half_bytes, spin_limit, ST(s)),
          "custom_allreduce_rmsnorm");
  });
  m.def("allreduce_buffer_alloc", [](long bytes, bool uncached) {
    uintptr_t p = 0;
    check(dab::allreduce_buffer_alloc(bytes, uncached ? 1 : 0, &p), "allreduce_buffer_alloc");
    return p;
  }, py::arg("bytes"), py::arg("uncached") = true);
  m.def("allreduce_buffer_free", [](u ptr) { check(dab::allreduce_buffer_free(ptr), "allreduce_buffer_free"); });
  m.def("ipc_get_handle", [](u ptr) {
    std::string h;
    check(dab::ipc_get_handle(ptr, &h), "ipc_get_handle");
    return py::bytes(h);
  });
  m.def("ipc_open_handle", [](const std::string& h) {
    uintptr_t p = 0;
    check(dab::ipc_open_handle(h, &p), "ipc_open_handle");
    return p;
  });
  m.def("ipc_probe", [](u ptr) { check(dab::ipc_probe(ptr), "ipc_probe"); });
  m.def("ipc_close_handle", [](u ptr) { check(dab::ipc_close_handle(ptr), "ipc_close_handle"); });
  m.def("allreduce_error", &dab::allreduce_error, py::arg("base"), py::arg("clear") = 1);
  m.def("allreduce_error_async", [](u base, u host_word, u s) {
    check(dab::allreduce_error_async(base, VP(host_word), ST(s)), "allreduce_error_async");
  });
  m.def("roctx_push", [](const std::string& name) { return dab::trace::range_push(name.c_str()); });
  m.def("roctx_pop", &dab::trace::range_pop);
  m.def("roctx_mark", [](const std::string& name) { dab::trace::mark(name.c_str()); });

  // ---------------- kernels ----------------
  m.def("rmsnorm", [](u out, u res_out, u x, u res_in, u w, int rows, int cols, float eps, u s) {
    check(dab::rmsnorm(VP(out), VP(res_out), CVP(x), CVP(res_in), CVP(w), rows, cols, eps, ST(s)), "rmsnorm");
  });
  m.def("layernorm", [](u out, u x, u res_in, u gamma, u beta, int rows, int cols, float eps, u s) {
    check(dab::layernorm(VP(out), CVP(x), CVP(res_in), CVP(gamma), CVP(beta), rows, cols, eps, ST(s)), "layernorm");
  });
  m.def("bert_embed", [](u out, u ids, u pos_ids, u type_ids, u word, u pos, u type, u gamma, u beta, int rows, int cols,
                         float eps, u s) {
    check(dab::bert_embed(VP(out), (const int*)ids, (const int*)pos_ids, (const int*)type_ids, CVP(word), CVP(pos),
                          CVP(type), CVP(gamma), CVP(beta), rows, cols, eps, ST(s)),
          "bert_embed");
  });
  m.def("embed_gather", [](u out, u ids, u table, int rows, int cols, u s) {
    check(dab::embed_gather(VP(out), (const int*)ids, CVP(table), rows, cols, ST(s)), "embed_gather");
  });
  m.def("mean_pool", [](u out, u out_bf16, u hidden, u cu, int batch, int cols, int normalize, u s) {
    check(dab::mean_pool((float*)out, VP(out_bf16), CVP(hidden), (const int*)cu, batch, cols, normalize, ST(s)),
          "mean_pool");
  });
  m.def("gelu", [](u out, u x, u bias, size_t rows, int cols, u s) {
    check(dab::gelu(VP(out), CVP(x), CVP(bias), rows, cols, ST(s)), "gelu");
  });
  m.def("silu_mul", [](u out, u x, size_t rows, int F, u s, int interleaved) {
    check(dab::silu_mul(VP(out), CVP(x), rows, F, ST(s), interleaved), "silu_mul");
  }, py::arg("out"), py::arg("x"), py::arg("rows"), py::arg("F"), py::arg("s"), py::arg("interleaved") = 0);
  m.def("rope_kv_write", [](u qkv, int ld, u positions, u cos_sin, u q_out, u k_cache, u v_cache, u slots, int T,
                            int Hq, int Hkv, int D, int block_size, u s, u slabs, int S, long slab_stride,
                            int slab_bf16) {
    check(dab::rope_kv_write(CVP(qkv), ld, (const int*)positions, CVP(cos_sin), VP(q_out), VP(k_cache), VP(v_cache),
                             (const int64_t*)slots, T, Hq, Hkv, D, block_size, ST(s), CVP(slabs), S, slab_stride,
                             slab_bf16),
          "rope_kv_write");
  }, py::arg("qkv"), py::arg("ld"), py::arg("positions"), py::arg("cos_sin"), py::arg("q_out"), py::arg("k_cache"),
     py::arg("v_cache"), py::arg("slots"), py::arg("T"), py::arg("Hq"), py::arg("Hkv"), py::arg("D"),
     py::arg("block_size"), py::arg("s"), py::arg("slabs") = 0, py::arg("S") = 0, py::arg("slab_stride") = 0,
     py::arg("slab_bf16") = 0);
  m.def("rmsnorm_slabs", [](u out, u res_out, u slabs, int S, long slab_stride, u res_in, u w, int rows, int cols,
                            float eps, u s, int slab_bf16) {
    check(dab::rmsnorm_slabs(VP(out), VP(res_out), CVP(slabs), S, slab_stride, CVP(res_in), CVP(w), rows, cols, eps,
                             ST(s), slab_bf16),
          "rmsnorm_slabs");
  }, py::arg("out"), py::arg("res_out"), py::arg("slabs"), py::arg("S"), py::arg("slab_stride"), py::arg("res_in"),
     py::arg("w"), py::arg("rows"), py::arg("cols"), py::arg("eps"), py::arg("s"), py::arg("slab_bf16") = 0);
  m.def("flash_attention",
        [](u q, long qst, long qsh, u k, u v, long kvst, long kvsh, u kc, u vc, u bt, int max_blocks, int bs, u out,
           long ost, long osh, u cu_q, u cu_k, u ctx_k, int batch, int max_sq, int Hq, int Hkv, int D, int causal,
           int paged, float scale, u s) {
          check(dab::flash_attention(CVP(q), qst, qsh, CVP(k), CVP(v), kvst, kvsh, CVP(kc), CVP(vc), (const int*)bt,
                                     max_blocks, bs, VP(out), ost, osh, (const int*)cu_q, (const int*)cu_k,
                                     (const int*)ctx_k, batch, max_sq, Hq, Hkv, D, causal, paged, scale, ST(s)),
                "flash_attention");
        });
  // Llama prefill attention with RoPE applied to Q on load (positions int32 [Tq], cos/sin table)
  m.def("flash_attention_rope",
        [](u q, long qst, long qsh, u kc, u vc, u bt, int max_blocks, int bs, u out, long ost, long osh, u cu_q,
           u ctx_k, int batch, int max_sq, int Hq, int Hkv, int D, int causal, float scale, u rope_pos, u rope_cs,
           u s) {
          check(dab::flash_attention(CVP(q), qst, qsh, nullptr, nullptr, 0, 0, CVP(kc), CVP(vc), (const int*)bt,
                                     max_blocks, bs, VP(out), ost, osh, (const int*)cu_q, nullptr, (const int*)ctx_k,
                                     batch, max_sq, Hq, Hkv, D, causal, 1, scale, ST(s), (const int*)rope_pos,
                                     CVP(rope_cs)),
                "flash_attention_rope");
        });
  // HIP stream restricted to a set of CUs (bit i of the mask words = CU i): lets a compute-bound
  // workload run beside a bandwidth-bound one on disjoint CUs (benchmarks/overlap_probe.py).  The
  // handle is wrapped by torch.cuda.ExternalStream; destroy it with destroy_stream.
  m.def("flash_attention_window",
        [](u q, long qst, long qsh, u k, u v, long kvst, long kvsh, u out, long ost, long osh, u cu_q, u cu_k,
           int batch, int max_sq, int H, int D, float scale, int window, u sink, u s) {
          check(dab::flash_attention(CVP(q), qst, qsh, CVP(k), CVP(v), kvst, kvsh, nullptr, nullptr, nullptr, 0, 0,
                                     VP(out), ost, osh, (const int*)cu_q, (const int*)cu_k, nullptr, batch, max_sq, H,
                                     H, D, 1, 0, scale, ST(s), nullptr, nullptr, window, (const float*)sink),
                "flash_attention_window");
        });
  m.def("embed_dyt", [](u x, u h, u ids, u table, int f32, float scale, float alpha, u w, u b, int rows, int cols, u s) {
    check(dab::embed_dyt((float*)x, VP(h), (const int*)ids, CVP(table), f32, scale, alpha, (const float*)w,
                         (const float*)b, rows, cols, ST(s)),
          "embed_dyt");
  });
  m.def("dyt_residual", [](u x, u h, int h_f32, u y, int y_f32, int S, long slab_stride, float a_post, u w_post,
                           u b_post, u ls, float a_next, u w_next, u b_next, int rows, int cols, u s) {
    check(dab::dyt_residual((float*)x, VP(h), h_f32, CVP(y), y_f32, S, slab_stride, a_post, (const float*)w_post,
                            (const float*)b_post, (const float*)ls, a_next, (const float*)w_next,
                            (const float*)b_next, rows, cols, ST(s)),
          "dyt_residual");
  });
  m.def("glu_f32", [](u out, long ldo, u x, long rows, int F, int act, u bias, u row_scale, u perm, int scale_in,
                      u s) {
    check(dab::glu_f32((float*)out, ldo, (const float*)x, rows, F, act, (const float*)bias, (const float*)row_scale,
                       (const int*)perm, scale_in, ST(s)),
          "glu_f32");
  });
  // chunked / sink attention over the paged cache
  m.def("flash_attention_chunk",
        [](u q, long qst, long qsh, u kc, u vc, u bt, int max_blocks, int bs, u out, long ost, long osh, u cu_q, u ctx_k,
           int batch, int max_sq, int Hq, int Hkv, int D, float scale, int chunk, u sink, u slopes, float out_scale,
           const std::tuple<u, int, int, long, long, int, int>& gate, u s) {
          const dab::OutputGate og{{CVP(std::get<0>(gate)), std::get<1>(gate), std::get<2>(gate), std::get<3>(gate), std::get<4>(gate)},
                                   std::get<5>(gate), std::get<6>(gate)};
          check(dab::flash_attention(CVP(q), qst, qsh, nullptr, nullptr, 0, 0, CVP(kc), CVP(vc), (const int*)bt,
                                     max_blocks, bs, VP(out), ost, osh, (const int*)cu_q, nullptr, (const int*)ctx_k,
                                     batch, max_sq, Hq, Hkv, D, 1, 1, scale, ST(s), nullptr, nullptr, 0,
                                     (const float*)sink, chunk, out_scale, (const float*)slopes, &og),
                "flash_attention_chunk");
        });
  m.def("any_attention", [](u q, u kc, u vc, int f32, u bt, int max_blocks, int bs, u cu, u ctx, int B, int T, int H,
                            int G, int D, int chunk, float scale, u sink, u slopes, u out, long o_tok, float out_scale,
                            u s) {
    check(dab::any_attention(CVP(q), CVP(kc), CVP(vc), f32, (const int*)bt, max_blocks, bs, (const int*)cu,
                             (const int*)ctx, B, T, H, G, D, chunk, scale, (const float*)sink, (const float*)slopes, VP(out), o_tok, out_scale,
                             ST(s)),
          "any_attention");
  });
  // a projection is passed as (pointer, fp32, slabs, slab stride, row stride)
  using P = std::tuple<u, int, int, long, long>;
  const auto proj = [](const P& t) {
    return dab::Proj{CVP(std::get<0>(t)), std::get<1>(t), std::get<2>(t), std::get<3>(t), std::get<4>(t)};
  };
  m.def("rms_residual", [proj](u x, u h, int act_f32, const P& y, u bias, u pairs, int top, u ids, u table,
                               int table_f32, u post, u gain, int n_true, float eps, int rows, int cols, int fresh, u s) {
    check(dab::rms_residual((float*)x, VP(h), act_f32, proj(y), (const float*)bias, CVP(pairs), top, (const int*)ids,
                            CVP(table), table_f32, (const float*)post, (const float*)gain, n_true, eps, rows, cols, fresh,
                            ST(s)),
          "rms_residual");
  });
  m.def("sigmoid_gate", [proj](const P& y, int col0, int per, u x, long ldx, int act_f32, int n, int T, u s) {
    check(dab::sigmoid_gate(proj(y), col0, per, VP(x), ldx, act_f32, n, T, ST(s)), "sigmoid_gate");
  });
  m.def("softcap", [proj](const P& y, float cap, u out, int n, int T, u s) {
    check(dab::softcap(proj(y), cap, (float*)out, n, T, ST(s)), "softcap");
  });
  m.def("qk_rope_write", [proj](const P& y, int col0, int H, int G, int D, int dim, int rot, u freq, float eps, int norm,
                                u positions, u slots, u q, u kc, u vc, int act_f32, int bs, int T, u s) {
    check(dab::qk_rope_write(proj(y), col0, H, G, D, dim, rot, (const double*)freq, eps, norm, (const int*)positions,
                             (const int64_t*)slots, VP(q), VP(kc), VP(vc), act_f32, bs, T, ST(s)),
          "qk_rope_write");
  });
  // routed = (expert rows, indices, weights, choices per token, experts); gate = (projection, column, bias);
  // depth = (results, weights, stride, n, keep, sum ahead, results in it)
  m.def("gated_residual", [proj](u src, u x, u h, int act_f32, const P& y, u ids, const std::tuple<u, u, u, int, int>& routed,
                                 const P& g, int g_col, u g_bias, u post, const std::tuple<u, u, long, int, int, u, int>& depth, u gain,
                                 int n_true, float eps, int rows, int cols, u s) {
    dab::GatedResidual p{};
    p.src = (const float*)src, p.x = (float*)x, p.h = VP(h), p.y = proj(y), p.ids = (const int*)ids;
    p.pairs = CVP(std::get<0>(routed)), p.idx = (const int*)std::get<1>(routed), p.wt = (const float*)std::get<2>(routed);
    p.top = std::get<3>(routed), p.experts = std::get<4>(routed);
    p.g = proj(g), p.g_col = g_col, p.g_bias = (const float*)g_bias, p.post = (const float*)post;
    p.depth = (float*)std::get<0>(depth), p.weights = (const float*)std::get<1>(depth), p.depth_stride = std::get<2>(depth);
    p.n = std::get<3>(depth), p.keep = std::get<4>(depth), p.ahead = (const float*)std::get<5>(depth), p.from = std::get<6>(depth);
    p.gain = (const float*)gain, p.inv_n = 1.f / n_true, p.eps = eps, p.cols = cols;
    check(dab::gated_residual(p, act_f32, rows, ST(s)), "gated_residual");
  });
  m.def("depth_ahead", [](u over, long stride, u w, int n, int m, u out, u s) {
    check(dab::depth_ahead((const float*)over, stride, (const float*)w, n, m, (float*)out, ST(s)), "depth_ahead");
  });
  m.def("poly_norm", [proj](const P& y, int n, int cols, float a, float b, float c, float e, float eps, u out, int act_f32, int T,
                            u s) {
    check(dab::poly_norm(proj(y), n, cols, a, b, c, e, eps, VP(out), act_f32, T, ST(s)), "poly_norm");
  });
  // heads = (H, G, D, dim, whole); conv = (taps, weights, ring, slots); rot = (dims, turns, factor); temp = (coef, every);
  // cache = (k, v, block size); mix = (first values, their width, mode, weight)
  m.def("attn_inputs", [proj](const P& y, int col0, const std::tuple<int, int, int, int, int>& heads, float eps, u gain, u bias,
                              const std::tuple<int, u, u, u>& conv, const std::tuple<int, u, float>& rot,
                              const std::tuple<float, int>& temp, u positions, u slots, u q, const std::tuple<u, u, int>& cache,
                              const std::tuple<u, int, int, float>& mix, u cu, int row0, int rows, int max_q, int act_f32, u s) {
    dab::AttnInputs p{};
    const int dim = std::get<3>(heads);
    p.y = proj(y), p.col0 = col0, p.H = std::get<0>(heads), p.G = std::get<1>(heads), p.D = std::get<2>(heads);
    p.whole = std::get<4>(heads), p.eps = eps, p.gain = (const float*)gain, p.bias = (const float*)bias;
    p.inv_q = 1.f / (p.whole ? p.H * dim : dim), p.inv_k = 1.f / (p.whole ? p.G * dim : dim);
    p.taps = std::get<0>(conv), p.conv = (const float*)std::get<1>(conv), p.ring = VP(std::get<2>(conv));
    p.slot = (const int*)std::get<3>(conv);
    p.rot = std::get<0>(rot), p.turns = (const double*)std::get<1>(rot), p.rot_mul = std::get<2>(rot);
    p.t_coef = std::get<0>(temp), p.t_every = std::get<1>(temp);
    p.positions = (const int*)positions, p.slots = (const int64_t*)slots, p.q = VP(q);
    p.kc = VP(std::get<0>(cache)), p.vc = VP(std::get<1>(cache)), p.bs = std::get<2>(cache);
    p.first = VP(std::get<0>(mix)), p.first_w = std::get<1>(mix), p.mix = std::get<2>(mix), p.lam = std::get<3>(mix);
    p.cu = (const int*)cu, p.row0 = row0;
    check(dab::attn_inputs(p, act_f32, rows, max_q, ST(s)), "attn_inputs");
  });
  m.def("recurrent_state_width", &dab::recurrent_state_width);
  m.def("short_conv", [proj](const P& y, int col0, int C, int taps, u w, u bias, u ring, u slot, u pos, u cu, int chunks,
                             int max_q, u out, int act_f32, u s) {
    check(dab::short_conv(proj(y), col0, C, taps, (const float*)w, (const float*)bias, VP(ring), (const int*)slot,
                          (const int*)pos, (const int*)cu, chunks, max_q, VP(out), act_f32, ST(s)),
          "short_conv");
  });
  m.def("short_conv_step", [proj](const P& y, int col0, int C, int taps, u w, u bias, u ring, u slot, u pos, int row0, int B,
                                  u out, int z_col, u z_out, int act_f32, u s) {
    check(dab::short_conv_step(proj(y), col0, C, taps, (const float*)w, (const float*)bias, VP(ring), (const int*)slot,
                               (const int*)pos, row0, B, VP(out), z_col, VP(z_out), act_f32, ST(s)),
          "short_conv_step");
  });
  m.def("selective_state_width", &dab::selective_state_width);
  m.def("narrow_rows", [proj](const P& z, u out, u low, int N, int R, int T, u s) {
    check(dab::narrow_rows(proj(z), (float*)out, VP(low), N, R, T, ST(s)), "narrow_rows");
  });
  // shape = (C, Np, rank, b_col, c_col, z_col)
  using SS = std::tuple<int, int, int, int, int, int>;
  const auto sel = [](const SS& t) {
    return dab::SelectiveShape{std::get<0>(t), std::get<1>(t), std::get<2>(t), std::get<3>(t), std::get<4>(t), std::get<5>(t)};
  };
  m.def("selective_scan", [proj, sel](u x, int act_f32, const SS& d, const P& dt, const P& bc, const P& y, u A, u dt_bias,
                                      u skip, u state, u slot, u pos, u cu, int chunks, int max_q, int segs, u ws, u out, u s) {
    check(dab::selective_scan(CVP(x), act_f32, sel(d), proj(dt), proj(bc), proj(y), (const float*)A, (const float*)dt_bias,
                              (const float*)skip, (float*)state, (const int*)slot, (const int*)pos, (const int*)cu, chunks,
                              max_q, segs, (float*)ws, VP(out), ST(s)),
          "selective_scan");
  });
  m.def("selective_segments", [sel](const SS& d, int chunks, int max_q) { return dab::selective_segments(sel(d), chunks, max_q); });
  m.def("selective_step", [proj, sel](u x, int act_f32, const SS& d, u dt_w, u low, const P& bc, u A, u dt_bias,
                                      u skip, u state, u slot, u pos, int row0, int B, u out, u s) {
    check(dab::selective_step(CVP(x), act_f32, sel(d), CVP(dt_w), CVP(low), proj(bc), (const float*)A, (const float*)dt_bias,
                              (const float*)skip, (float*)state, (const int*)slot, (const int*)pos, row0, B, VP(out), ST(s)),
          "selective_step");
  });
  // shape = (delta, H, G, D, Dp, V, C, q_col, k_col, v_col, a_col, b_col)
  using R = std::tuple<int, int, int, int, int, int, int, int, int, int, int, int>;
  const auto shape = [](const R& t) {
    return dab::RecurrentShape{std::get<0>(t), std::get<1>(t), std::get<2>(t), std::get<3>(t), std::get<4>(t),  std::get<5>(t),
                               std::get<6>(t), std::get<7>(t), std::get<8>(t), std::get<9>(t), std::get<10>(t), std::get<11>(t)};
  };
  m.def("state_scan", [proj, shape](u conv, int act_f32, const R& d, const P& gates, u A, u dt_bias, u skip, u state,
                                    u slot, u pos, u cu, int chunks, u out, u s) {
    check(dab::state_scan(CVP(conv), act_f32, shape(d), proj(gates), (const float*)A, (const float*)dt_bias,
                          (const float*)skip, (float*)state, (const int*)slot, (const int*)pos, (const int*)cu, chunks,
                          VP(out), ST(s)),
          "state_scan");
  });
  m.def("state_chunks_ok", [shape](const R& d) { return dab::state_chunks_ok(shape(d)) != 0; });
  m.def("state_chunks_segments", [shape](const R& d, int chunks, int max_q) { return dab::state_chunks_segments(shape(d), chunks, max_q); });
  m.def("state_chunks_bytes", [shape](const R& d, int T, int chunks, int segs) { return dab::state_chunks_bytes(shape(d), T, chunks, segs); });
  m.def("state_chunks", [proj, shape](u conv, const R& d, const P& gates, u A, u dt_bias, u skip, u state, u slot, u pos,
                                      u cu, int chunks, int max_q, int T, int segs, u out, u ws, u s) {
    check(dab::state_chunks(CVP(conv), shape(d), proj(gates), (const float*)A, (const float*)dt_bias, (const float*)skip,
                            (float*)state, (const int*)slot, (const int*)pos, (const int*)cu, chunks, max_q, T, segs,
                            VP(out), VP(ws), ST(s)),
          "state_chunks");
  });
  m.def("state_decode", [proj, shape](const P& y, int col0, int taps, u w, u bias, u ring, int act_f32, const R& d,
                                      const P& gates, u A, u dt_bias, u skip, u state, u slot, u pos, int row0, int B,
                                      int g_col, u norm, float eps, float out_scale, u out, long ldo, int pad, u s) {
    check(dab::state_decode(proj(y), col0, taps, (const float*)w, (const float*)bias, VP(ring), act_f32, shape(d),
                            proj(gates), (const float*)A, (const float*)dt_bias, (const float*)skip, (float*)state,
                            (const int*)slot, (const int*)pos, row0, B, g_col, (const float*)norm, eps, out_scale,
                            VP(out), ldo, pad, ST(s)),
          "state_decode");
  });
  m.def("gated_norm", [proj](u y, int act_f32, const P& gate, int g_col, int n, int part, int gate_first, int per_head,
                             u w, float eps, float scale, u out, long ldo, int pad, int row0, int T, u s) {
    check(dab::gated_norm(CVP(y), act_f32, proj(gate), g_col, n, part, gate_first, per_head, (const float*)w, eps, scale,
                          VP(out), ldo, pad, row0, T, ST(s)),
          "gated_norm");
  });
  m.def("moe_route", [proj](const P& z, int col0, int E, int top, float scale, int scores, u correction, u idx, u wt, int T,
                            u s) {
    check(dab::moe_route(proj(z), col0, E, top, scale, scores, (const float*)correction, (int*)idx, (float*)wt, T, ST(s)), "moe_route");
  });
  m.def("moe_plan_words", &dab::moe_plan_words);
  m.def("moe_plan", [](u idx, int pairs, int E, int bm, u perm, u tiles, int max_tiles, u ws, u s) {
    check(dab::moe_plan((const int*)idx, pairs, E, bm, (int*)perm, VP(tiles), max_tiles, (int*)ws, ST(s)), "moe_plan");
  });
  m.def("shared_glu", [proj](const P& y, int col0, int F, const P& z, int sg_col, u out, long ldo, int act_f32, int T, u s) {
    check(dab::shared_glu(proj(y), col0, F, proj(z), sg_col, VP(out), ldo, act_f32, T, ST(s)), "shared_glu");
  });
  m.def("gemm_narrow", [](u A, long lda, u B, u C, int M, int N, int K, int S, int tall, u s) {
    check(dab::gemm_narrow(CVP(A), lda, CVP(B), (float*)C, M, N, K, S, tall, ST(s)), "gemm_narrow");
  });
  m.def("gemm_grouped", [](u A, long lda, u B, u C, long ldc, int N, int K, u perm, int a_div, int scatter, u tiles,
                           int n_tiles, int bm, int glu, u row_scale, int scale_in, u s) {
    check(dab::gemm_grouped(CVP(A), lda, CVP(B), VP(C), ldc, N, K, (const int*)perm, a_div, scatter, CVP(tiles), n_tiles,
                            bm, glu, (const float*)row_scale, scale_in, ST(s)),
          "gemm_grouped");
  });
  m.def("gemm_f32_grouped", [](u A, long lda, u B, u C, long ldc, int N, int K, u perm, int a_div, int scatter, u tiles,
                               int n_tiles, u s) {
    check(dab::gemm_f32_grouped((const float*)A, lda, (const float*)B, (float*)C, ldc, N, K, (const int*)perm, a_div,
                                scatter, CVP(tiles), n_tiles, ST(s)),
          "gemm_f32_grouped");
  });
  m.def("gemm_f32", [](u A, long lda, long sa, u B, long ldb, long sb, u C, long ldc, long sc, int M, int N, int K,
                       int batch, u s) {
    check(dab::gemm_f32((const float*)A, lda, sa, (const float*)B, ldb, sb, (float*)C, ldc, sc, M, N, K, batch, ST(s)),
          "gemm_f32");
  });
  m.def("latent_write", [](u y, int y_f32, int S, long slab_stride, long ld, u q_out, int q_cols, u gain, u cache,
                           int cache_f32, u slots, int T, int R, int rank, float eps,
                           const std::tuple<u, u, int, int, int, int, float>& rope, u s) {
    const auto& [freq, positions, rot, D, q_at, c_at, mul] = rope;
    check(dab::latent_write(CVP(y), y_f32, S, slab_stride, ld, VP(q_out), q_cols, (const float*)gain, VP(cache),
                            cache_f32, (const int64_t*)slots, T, R, rank, eps,
                            dab::LatentRope{(const double*)freq, (const int*)positions, rot, D, q_at, c_at, mul}, ST(s)),
          "latent_write");
  });
  m.def("latent_gather", [](u out, u cache, u bt, int max_blocks, int bs, u cu_k, u ctx, int B, int total,
                            int row_bytes, u s) {
    check(dab::latent_gather(VP(out), CVP(cache), (const int*)bt, max_blocks, bs, (const int*)cu_k, (const int*)ctx, B,
                             total, row_bytes, ST(s)),
          "latent_gather");
  });
  m.def("head_gemm", [](u y, long y_tok, long y_head, u x, long x_tok, long x_head, u w, int row0, int T, int H, int N,
                        int K, u s) {
    check(dab::head_gemm(VP(y), y_tok, y_head, CVP(x), x_tok, x_head, CVP(w), row0, T, H, N, K, ST(s)), "head_gemm");
  });
  m.def("latent_key_fill", [](u k, long k_tok, int D, u rows, int R, int q_at, int c_at, int rot, int H, int T, u s) {
    check(dab::latent_key_fill(VP(k), k_tok, D, CVP(rows), R, q_at, c_at, rot, H, T, ST(s)), "latent_key_fill");
  });
  m.def("latent_decode_ok", &dab::latent_decode_ok);
  m.def("latent_decode_values", &dab::latent_decode_values);
  m.def("latent_decode_groups", &dab::latent_decode_groups);
  m.def("latent_decode", [](u q, u cache, u bt, int max_blocks, int bs, u ctx, u sink, u out, u po, u pml, int B,
                            int H, int R, int window, int parts, int min_part, float scale, u order, u s) {
    check(dab::latent_decode(CVP(q), CVP(cache), (const int*)bt, max_blocks, bs, (const int*)ctx, (const float*)sink,
                             VP(out), (float*)po, (float*)pml, B, H, R, window, parts, min_part, scale,
                             (const int*)order, ST(s)),
          "latent_decode");
  });
  m.def("latent_any", [](u out, u q, u cache, int f32, u bt, int max_blocks, int bs, u cu_q, u ctx, int B, u sink,
                         int T, int H, int R, int window, float scale, u s) {
    check(dab::latent_any(VP(out), CVP(q), CVP(cache), f32, (const int*)bt, max_blocks, bs, (const int*)cu_q,
                          (const int*)ctx, B, (const float*)sink, T, H, R, window, scale, ST(s)),
          "latent_any");
  });
  m.def("create_cu_masked_stream", [](std::vector<uint32_t> mask) {
    hipStream_t st = nullptr;
    check(hipExtStreamCreateWithCUMask(&st, (uint32_t)mask.size(), mask.data()), "hipExtStreamCreateWithCUMask");
    return reinterpret_cast<uintptr_t>(st);
  });
  m.def("destroy_stream", [](u s) { check(hipStreamDestroy(ST(s)), "hipStreamDestroy"); });
  m.def("paged_decode_attention", [](u q, u kc, u vc, u bt, int max_blocks, int bs, u ctx, u out, u po, u pm, u pl,
                                     u cnt, int batch, int Hq, int Hkv, int D, int part_size, int max_parts,
                                     float scale, u s, u order, u w0, long w0_bytes, u w1, long w1_bytes,
                                     int w_blocks, int chunk, u sink, float out_scale, long o_stride, u slopes,
                                     const std::tuple<u, int, int, long, long, int, int>& gate) {
    dab::L3Warm warm{{(const char*)w0, (const char*)w1}, {w0_bytes, w1_bytes}, w_blocks};
    // gate = (projection, column, columns of the output it covers each)
    const dab::OutputGate og{{CVP(std::get<0>(gate)), std::get<1>(gate), std::get<2>(gate), std::get<3>(gate), std::get<4>(gate)},
                             std::get<5>(gate), std::get<6>(gate)};
    check(dab::paged_decode_attention(CVP(q), CVP(kc), CVP(vc), (const int*)bt, max_blocks, bs, (const int*)ctx, VP(out),
                                      (float*)po, (float*)pm, (float*)pl, (int*)cnt, batch, Hq, Hkv, D, part_size,
                                      max_parts, scale, ST(s), (const int*)order, &warm, chunk, (const float*)sink,
                                      out_scale, o_stride, (const float*)slopes, &og),
          "paged_decode_attention");
  }, py::arg("q"), py::arg("kc"), py::arg("vc"), py::arg("bt"), py::arg("max_blocks"), py::arg("bs"), py::arg("ctx"),
     py::arg("out"), py::arg("po"), py::arg("pm"), py::arg("pl"), py::arg("cnt"), py::arg("batch"), py::arg("Hq"),
     py::arg("Hkv"), py::arg("D"), py::arg("part_size"), py::arg("max_parts"), py::arg("scale"), py::arg("s"),
     py::arg("order") = 0, py::arg("w0") = 0, py::arg("w0_bytes") = 0, py::arg("w1") = 0, py::arg("w1_bytes") = 0,
     py::arg("w_blocks") = 0, py::arg("chunk") = 0, py::arg("sink") = 0, py::arg("out_scale") = 1.f,
     py::arg("o_stride") = 0, py::arg("slopes") = 0,
     py::arg("gate") = std::make_tuple((u)0, 0, 1, 0L, 0L, 0, 1));
  m.def("gemm_bt", [](u A, long lda, u B, long ldb, u C, long ldc, u bias, u residual, long ldr, int M, int N, int K,
                      int epilogue, int out_f32, u row_group, u q_group, u allow, int allow_words, u s, int b_rows,
                      int b_group) {
    check(dab::gemm_bt(CVP(A), lda, CVP(B), ldb, VP(C), ldc, CVP(bias), CVP(residual), ldr, M, N, K, epilogue, out_f32,
                       (const int*)row_group, (const int*)q_group, (const uint32_t*)allow, allow_words, ST(s), b_rows,
                       b_group),
          "gemm_bt");
  }, py::arg("A"), py::arg("lda"), py::arg("B"), py::arg("ldb"), py::arg("C"), py::arg("ldc"), py::arg("bias"),
     py::arg("residual"), py::arg("ldr"), py::arg("M"), py::arg("N"), py::arg("K"), py::arg("epilogue"),
     py::arg("out_f32"), py::arg("row_group"), py::arg("q_group"), py::arg("allow"), py::arg("allow_words"),
     py::arg("s"), py::arg("b_rows") = 0, py::arg("b_group") = 1);
  m.def("gemm_mid_ok", &dab::gemm_mid_ok);
  m.def("gemm_mid_slab_bytes", &dab::gemm_mid_slab_bytes);
  m.def("gemm_mid_counters", &dab::gemm_mid_counters);
  m.def("gemm_mid", [](u A, long lda, u B, u C, long ldc, u residual, long ldr, int M, int N, int K, int epilogue,
                       u slabs, long slab_bytes, u cnt, int n_cnt, u s, int variant, int b_group) {
    check(dab::gemm_mid(CVP(A), lda, CVP(B), VP(C), ldc, CVP(residual), ldr, M, N, K, epilogue, VP(slabs), slab_bytes,
                        (int*)cnt, n_cnt, ST(s), variant, b_group),
          "gemm_mid");
  }, py::arg("A"), py::arg("lda"), py::arg("B"), py::arg("C"), py::arg("ldc"), py::arg("residual"), py::arg("ldr"),
     py::arg("M"), py::arg("N"), py::arg("K"), py::arg("epilogue"), py::arg("slabs"), py::arg("slab_bytes"),
     py::arg("cnt"), py::arg("n_cnt"), py::arg("s"), py::arg("variant") = 0, py::arg("b_group") = 1);
  m.def("gemm256_ok", &dab::gemm256_ok);
  m.def("gemm256_stamped", [](u A, long lda, u B, u C, u bias, u residual, int M, int N, int K, int epilogue,
                              int b_shuf, u stamps, int stamp_tiles, u s, int store_aux) {
    const int r = dab::gemm256_stamped(CVP(A), lda, CVP(B), VP(C), CVP(bias), CVP(residual), M, N, K, epilogue, b_shuf,
                                       VP(stamps), stamp_tiles, ST(s), store_aux);
    if (r < 0) check(-r, "gemm256_stamped");
    return r;
  }, py::arg("A"), py::arg("lda"), py::arg("B"), py::arg("C"), py::arg("bias"), py::arg("residual"), py::arg("M"),
     py::arg("N"), py::arg("K"), py::arg("epilogue"), py::arg("b_shuf"), py::arg("stamps"), py::arg("stamp_tiles"),
     py::arg("s"), py::arg("store_aux") = 0);
  m.def("gemm256_candidates_stamped", [](u A, long lda, u B, int M, int N, int K, int b_rows, u thr, u cnt, u cand_val,
                                          u cand_idx, int cap, u stamps, int stamp_tiles, u s) {
    const int r = dab::gemm256_candidates_stamped(CVP(A), lda, CVP(B), M, N, K, b_rows, (const float*)thr, (int*)cnt,
                                                  (float*)cand_val, (int*)cand_idx, cap, VP(stamps), stamp_tiles, ST(s));
    if (r < 0) check(-r, "gemm256_candidates_stamped");
    return r;
  });
  m.def("gemm256", [](u A, long lda, u B, long ldb, u C, long ldc, u bias, u residual, long ldr, int M, int N, int K,
                      int epilogue, u s, int b_shuf, int b_group) {
    check(dab::gemm256(CVP(A), lda, CVP(B), ldb, VP(C), ldc, CVP(bias), CVP(residual), ldr, M, N, K, epilogue, ST(s),
                       b_shuf, b_group),
          "gemm256");
  }, py::arg("A"), py::arg("lda"), py::arg("B"), py::arg("ldb"), py::arg("C"), py::arg("ldc"), py::arg("bias"),
     py::arg("residual"), py::arg("ldr"), py::arg("M"), py::arg("N"), py::arg("K"), py::arg("epilogue"), py::arg("s"),
     py::arg("b_shuf") = 0, py::arg("b_group") = 1);
  m.def("gemm_score_candidates", [](u A, long lda, u B, long ldb, int M, int N, int K, u row_group, u q_group, u thr,
                                    u cnt, u cand_val, u cand_idx, int cap, u s) {
    check(dab::gemm_score_candidates(CVP(A), lda, CVP(B), ldb, M, N, K, reinterpret_cast<const int*>(row_group),
                                     reinterpret_cast<const int*>(q_group), reinterpret_cast<const float*>(thr),
                                     reinterpret_cast<int*>(cnt), reinterpret_cast<float*>(cand_val),
                                     reinterpret_cast<int*>(cand_idx), cap, ST(s)),
          "gemm_score_candidates");
  });
  // candidates over a shuffle_weights copy of the rows (b_rows of them): 1..16 queries on the
  // persistent scan, 17..128 on the weight-streaming kernel, more on the 8-phase GEMM
  m.def("score_candidates_shuf", [](u A, long lda, u Wshuf, int M, int N, int K, u row_group, u q_group, u thr,
                                    u cnt, u cand_val, u cand_idx, int cap, u s, int b_rows) {
    auto* rg = reinterpret_cast<const int*>(row_group);
    auto* qg = reinterpret_cast<const int*>(q_group);
    auto* th = reinterpret_cast<const float*>(thr);
    auto* ct = reinterpret_cast<int*>(cnt);
    auto* cv = reinterpret_cast<float*>(cand_val);
    auto* ci = reinterpret_cast<int*>(cand_idx);
    int rc = hipErrorInvalidValue;
    if (K % 256 == 0 && ((M <= 64 && K <= 1024) || (M <= 96 && K <= 768)))
      rc = dab::index_scan_candidates_shuf(CVP(A), lda, CVP(Wshuf), M, N, K, rg, qg, th, ct, cv, ci, cap, ST(s));
    else if (M <= 64 || K % 128)
      rc = dab::stream_score_candidates_shuf(CVP(A), lda, CVP(Wshuf), M, N, K, rg, qg, th, ct, cv, ci, cap, ST(s));
    else  // 65+ queries past the scan's limits: the persistent 256x256 kernel (gemm256 G_CAND); at
          // 97-127 queries of 768 the streaming kernel took 5.6-6.0 ms on 10M rows, gemm256 ~3.9
      rc = dab::gemm_score_candidates(CVP(A), lda, CVP(Wshuf), K, M, N, K, rg, qg, th, ct, cv, ci, cap, ST(s), b_rows);
    check(rc, "score_candidates_shuf");
  }, py::arg("A"), py::arg("lda"), py::arg("Wshuf"), py::arg("M"), py::arg("N"), py::arg("K"), py::arg("row_group"),
     py::arg("q_group"), py::arg("thr"), py::arg("cnt"), py::arg("cand_val"), py::arg("cand_idx"), py::arg("cap"),
     py::arg("s"), py::arg("b_rows") = 0);
  m.def("stream_gemm", [](u X, long ldx, u W, long ldw, u out, long ldo, u residual, long ldr, int M, int N, int K,
                          int S, int epilogue, u s, int nt, int cfg, float norm_eps, int slab_bf16, int w_group) {
    check(dab::stream_gemm(CVP(X), ldx, CVP(W), ldw, VP(out), ldo, CVP(residual), ldr, M, N, K, S, epilogue, ST(s), nt,
                           cfg, norm_eps, slab_bf16, w_group),
          "stream_gemm");
  }, py::arg("X"), py::arg("ldx"), py::arg("W"), py::arg("ldw"), py::arg("out"), py::arg("ldo"), py::arg("residual"),
     py::arg("ldr"), py::arg("M"), py::arg("N"), py::arg("K"), py::arg("S"), py::arg("epilogue"), py::arg("s"),
     py::arg("nt"), py::arg("cfg"), py::arg("norm_eps") = 0.f, py::arg("slab_bf16") = 0, py::arg("w_group") = 1);
  m.def("stream_gemm_bn", &dab::stream_gemm_bn);
  m.def("stream_gemm_max_m", &dab::stream_gemm_max_m);
  m.def("stream_gemm_set_slice_xcd", &dab::stream_gemm_set_slice_xcd);
  m.def("stream_gemm_slice_xcd", &dab::stream_gemm_slice_xcd);
  m.def("stream_gemm_shuffled", &dab::stream_gemm_shuffled);
  m.def("slab_reduce", [](u out, long ldo, u slabs, int S, int M, int N, u residual, long ldr, u s, int slab_bf16) {
    check(dab::slab_reduce(VP(out), ldo, CVP(slabs), S, M, N, CVP(residual), ldr, ST(s), slab_bf16), "slab_reduce");
  }, py::arg("out"), py::arg("ldo"), py::arg("slabs"), py::arg("S"), py::arg("M"), py::arg("N"), py::arg("residual"),
     py::arg("ldr"), py::arg("s"), py::arg("slab_bf16") = 0);
  m.def("sample_tokens", [](u logits, int f32, long ld, int rows, int vocab, u temp, u top_k, u top_p,
                            unsigned long long seed, u counters, u out_tokens, u out_logprobs, u s) {
    check(dab::sample_tokens(CVP(logits), f32, ld, rows, vocab, (const float*)temp, (const int*)top_k,
                             (const float*)top_p, seed, (int64_t*)counters, (int*)out_tokens, (float*)out_logprobs,
                             ST(s)),
          "sample_tokens");
  });
  m.def("topk_rows", [](u scores, long ld, int rows, int n, int k, u out_vals, u out_idx, long long base, u out_idx64,
                        u s) {
    check(dab::topk_rows((const float*)scores, ld, rows, n, k, (float*)out_vals, (int*)out_idx, base,
                         (int64_t*)out_idx64, ST(s)),
          "topk_rows");
  });

  m.def("sample_tokens_2stage", [](u logits, int f32, long ld, int rows, int vocab, u temp, u top_k, u top_p,
                                   unsigned long long seed, u counters, u out_tokens, u ws, size_t ws_bytes, u s) {
    check(dab::sample_tokens_2stage(CVP(logits), f32, ld, rows, vocab, (const float*)temp, (const int*)top_k,
                                    (const float*)top_p, seed, (int64_t*)counters, (int*)out_tokens, VP(ws), ws_bytes,
                                    ST(s)),
          "sample_tokens_2stage");
  });
  m.def("mask_logits", [](u logits, int f32, long ld, int rows, int vocab, u mask, int words, u row_flags, u s,
                          long mask_ld) {
    check(dab::mask_logits(VP(logits), f32, ld, rows, vocab, (const uint32_t*)mask, words, (const int*)row_flags,
                           ST(s), mask_ld),
          "mask_logits");
  });
  m.def("sample_candidates", [](u logits, int f32, long ld, int rows, int vocab, int base, u keys, u idx, int ncand,
                                u s) {
    check(dab::sample_candidates(CVP(logits), f32, ld, rows, vocab, base, (uint32_t*)keys, (int*)idx, ncand, ST(s)),
          "sample_candidates");
  });
  m.def("sample_merge", [](u keys, u idx, int ncand, int rows, int vocab, u temp, u top_k, u top_p,
                           unsigned long long seed, u counters, u out_tokens, u s) {
    check(dab::sample_merge((const uint32_t*)keys, (const int*)idx, ncand, rows, vocab, (const float*)temp,
                            (const int*)top_k, (const float*)top_p, seed, (int64_t*)counters, (int*)out_tokens, ST(s)),
          "sample_merge");
  });
  m.def("topk_rows_2stage", [](u scores, long ld, int rows, int n, int k, u out_vals, u out_idx, long long base,
                               u out_idx64, u ws, size_t ws_bytes, u s) {
    check(dab::topk_rows_2stage((const float*)scores, ld, rows, n, k, (float*)out_vals, (int*)out_idx, base,
                                (int64_t*)out_idx64, VP(ws), ws_bytes, ST(s)),
          "topk_rows_2stage");
  });

  // ---------------- tokenizer ----------------
  py::class_<dab::TokenizerConfig>(m, "TokenizerConfig")
      .def(py::init<>())
      .def_readwrite("vocab_size", &dab::TokenizerConfig::vocab_size)
      .def_readwrite("first_id", &dab::TokenizerConfig::first_id)
      .def_readwrite("last_id", &dab::TokenizerConfig::last_id)
      .def_readwrite("pad_id", &dab::TokenizerConfig::pad_id)
      .def_readwrite("unk_id", &dab::TokenizerConfig::unk_id)
      .def_readwrite("cls_id", &dab::TokenizerConfig::cls_id)
      .def_readwrite("sep_id", &dab::TokenizerConfig::sep_id)
      .def_readwrite("max_word_chars", &dab::TokenizerConfig::max_word_chars);
  py::class_<dab::HashTokenizer>(m, "HashTokenizer")
      .def(py::init<const dab::TokenizerConfig&>())
      .def("encode", &dab::HashTokenizer::encode, py::arg("text"), py::arg("add_special") = true,
           py::arg("max_len") = 0)
      .def(
          "encode_batch",
          [](const dab::HashTokenizer& t, const std::vector<std::string>& texts, bool add_special, int max_len,
             int threads) {
            std::vector<int32_t> ids;
            std::vector<int64_t> offs;
            {
              py::gil_scoped_release rel;
              t.encode_batch(texts, add_special, max_len, threads, ids, offs);
            }
            py::array_t<int32_t> a(ids.size());
            std::copy(ids.begin(), ids.end(), a.mutable_data());
            py::array_t<int64_t> o(offs.size());
            std::copy(offs.begin(), offs.end(), o.mutable_data());
            return py::make_tuple(a, o);
          },
          py::arg("texts"), py::arg("add_special") = true, py::arg("max_len") = 0, py::arg("threads") = 8)
      .def("decode", &dab::HashTokenizer::decode, py::arg("ids"), py::arg("skip_special") = true)
      .def("token_texts",
           [](const dab::HashTokenizer& t) {
             py::list out;
             for (const auto& w : t.token_texts()) out.append(py::bytes(w));
             return out;
           })
      .def_static("count_words", &dab::HashTokenizer::count_words);

  // ---------------- JSON-constrained decoding ----------------
  py::class_<dab::JsonVocab, std::shared_ptr<dab::JsonVocab>>(m, "JsonVocab")
      .def(py::init([](const std::vector<py::bytes>& toks, const std::vector<int32_t>& eos) {
             std::vector<std::string> t;
             t.reserve(toks.size());
             for (const auto& b : toks) t.emplace_back(b);
             return std::make_shared<dab::JsonVocab>(t, eos);
           }),
           py::arg("tokens"), py::arg("eos_ids"))
      .def("vocab_size", &dab::JsonVocab::vocab_size)
      .def("words", &dab::JsonVocab::words)
      .def("trie_nodes", &dab::JsonVocab::trie_nodes)
      .def("cache_entries", &dab::JsonVocab::cache_entries);
  py::class_<dab::JsonMatcher>(m, "JsonMatcher")
      .def(py::init<std::shared_ptr<dab::JsonVocab>, int, int>(), py::arg("vocab"), py::arg("max_depth") = 24,
           py::arg("max_ws") = 8)
      .def("fill_mask",
           [](dab::JsonMatcher& j, int remaining, u out) {
             py::gil_scoped_release rel;
             return j.fill_mask(remaining, (uint32_t*)out);
           })
      .def("advance", &dab::JsonMatcher::advance)
      .def("done", &dab::JsonMatcher::done)
      .def("broken", &dab::JsonMatcher::broken)
      .def("completion", [](const dab::JsonMatcher& j) { return py::bytes(j.completion()); })
      .def("completion_len", &dab::JsonMatcher::completion_len)
      .def("text", [](const dab::JsonMatcher& j) { return py::bytes(j.text()); });
  py::class_<dab::SchemaAutomaton, std::shared_ptr<dab::SchemaAutomaton>>(m, "SchemaAutomaton")
      .def(py::init<std::shared_ptr<dab::JsonVocab>, int, int, const std::vector<int32_t>&,
                    const std::vector<std::vector<int32_t>>&, const std::vector<std::vector<int32_t>>&>(),
           py::arg("vocab"), py::arg("n_states"), py::arg("start"), py::arg("accept"), py::arg("edges"),
           py::arg("eps"))
      .def("dfa_states", &dab::SchemaAutomaton::dfa_states)
      .def("accepts", [](dab::SchemaAutomaton& a, const py::bytes& b) {
        int d = a.start();
        for (unsigned char c : std::string(b)) {
          d = a.step(d, c);
          if (d < 0) return false;
        }
        return a.accepting(d);
      });
  py::class_<dab::SchemaMatcher>(m, "SchemaMatcher")
      .def(py::init<std::shared_ptr<dab::SchemaAutomaton>>(), py::arg("automaton"))
      .def("fill_mask",
           [](dab::SchemaMatcher& j, int remaining, u out) {
             py::gil_scoped_release rel;
             return j.fill_mask(remaining, (uint32_t*)out);
           })
      .def("advance", &dab::SchemaMatcher::advance)
      .def("done", &dab::SchemaMatcher::done)
      .def("broken", &dab::SchemaMatcher::broken)
      .def("completion_len", &dab::SchemaMatcher::completion_len)
      .def("text", [](const dab::SchemaMatcher& j) { return py::bytes(j.text()); });
  m.def("json_accepts", [](const py::bytes& b, bool complete, int max_depth, int max_ws) {
    return dab::json_accepts(std::string(b), complete, max_depth, max_ws);
  }, py::arg("bytes"), py::arg("complete") = true, py::arg("max_depth") = 64, py::arg("max_ws") = 255);

  // ---------------- KV block manager ----------------
  py::class_<dab::KVBlockManager>(m, "KVBlockManager")
      .def(py::init<int, int, bool, int>(), py::arg("num_blocks"), py::arg("block_size"), py::arg("prefix_cache") = true,
           py::arg("state_slots") = 0)
      .def("add_sequence", &dab::KVBlockManager::add_sequence)
      .def("extend", &dab::KVBlockManager::extend)
      .def("append_tokens", &dab::KVBlockManager::append_tokens)
      .def("commit_prefix", &dab::KVBlockManager::commit_prefix)
      .def("free_sequence", &dab::KVBlockManager::free_sequence)
      .def("has", &dab::KVBlockManager::has)
      .def("num_tokens", &dab::KVBlockManager::num_tokens)
      .def("capacity_tokens", &dab::KVBlockManager::capacity_tokens)
      .def("num_free_blocks", &dab::KVBlockManager::num_free_blocks)
      .def("num_blocks", &dab::KVBlockManager::num_blocks)
      .def("block_size", &dab::KVBlockManager::block_size)
      .def("prefix_hits", &dab::KVBlockManager::prefix_hits)
      .def("blocks", &dab::KVBlockManager::blocks)
      .def("num_free_state_slots", &dab::KVBlockManager::num_free_state_slots)
      .def("state_slots_into", [](const dab::KVBlockManager& k, const std::vector<int64_t>& seqs,
                                  u out) { k.state_slots(seqs, (int32_t*)out); })
      .def("slot_mapping_into",
           [](const dab::KVBlockManager& k, int64_t seq, int start, int n, u out) {
             k.slot_mapping(seq, start, n, (int64_t*)out);
           })
      .def("prepare_decode_into",
           [](dab::KVBlockManager& k, const std::vector<int64_t>& seqs, const std::vector<int32_t>& toks,
              int max_blocks, u ids, u pos, u slots, u ctx, u bt) {
             return k.prepare_decode(seqs, toks, max_blocks, (int32_t*)ids, (int32_t*)pos, (int64_t*)slots,
                                     (int32_t*)ctx, (int32_t*)bt);
           })
      .def("block_table_into", [](const dab::KVBlockManager& k, const std::vector<int64_t>& seqs, int max_blocks,
                                  u out) { k.block_table(seqs, max_blocks, (int32_t*)out); });

  // ---------------- retrieval post-processing ----------------
  m.def(
      "aggregate_documents",
      [](py::array_t<float, py::array::c_style | py::array::forcecast> dist,
         py::array_t<int64_t, py::array::c_style | py::array::forcecast> doc_ids, int max_scores_n, int top_n) {
        if (dist.size() != doc_ids.size()) throw std::invalid_argument("distances / doc_ids length mismatch");
        auto r = dab::aggregate_documents(dist.data(), doc_ids.data(), (int)dist.size(), max_scores_n, top_n);
        py::list out;
        for (auto& d : r) out.append(py::make_tuple(d.doc_id, d.score));
        return out;
      },
      py::arg("distances"), py::arg("doc_ids"), py::arg("max_scores_n"), py::arg("top_n"));
  m.def(
      "merge_topk",
      [](py::array_t<float, py::array::c_style | py::array::forcecast> vals,
         py::array_t<int64_t, py::array::c_style | py::array::forcecast> ids, int k_out) {
        if (vals.ndim() != 2 || ids.ndim() != 2 || vals.shape(0) != ids.shape(0) || vals.shape(1) != ids.shape(1))
          throw std::invalid_argument("vals / ids must be [S, k] arrays of the same shape");
        const int S = (int)vals.shape(0), k = (int)vals.shape(1);
        py::array_t<float> ov(k_out);
        py::array_t<int64_t> oi(k_out);
        dab::merge_topk(vals.data(), ids.data(), S, k, k_out, ov.mutable_data(), oi.mutable_data());
        return py::make_tuple(ov, oi);
      },
      py::arg("vals"), py::arg("ids"), py::arg("k_out"));
}
