// Bindings of the kernels of models with mixed layer kinds (hybrid_launchers.h).  Launch
// arguments cross as a dict: addresses and sizes by the field names of the argument structs.
#include <pybind11/pybind11.h>

#include "hybrid_launchers.h"

namespace py = pybind11;
using u64 = std::uintptr_t;

namespace {

template <class T>
T* P(u64 p) { return reinterpret_cast<T*>(p); }
hipStream_t S(u64 s) { return reinterpret_cast<hipStream_t>(s); }

struct Fields {
  const py::dict& d;
  template <class T>
  void ptr(const char* k, T*& out) const {
    if (d.contains(k)) out = reinterpret_cast<T*>(d[k].cast<u64>());
  }
  template <class T>
  void val(const char* k, T& out) const { out = d[k].cast<T>(); }
};

#define PTR(n) f.ptr(#n, a.n)
#define VAL(n) f.val(#n, a.n)

drtc::DeltaArgs delta_args(const py::dict& d) {
  const Fields f{d};
  drtc::DeltaArgs a{};
  PTR(proj); VAL(ldp); VAL(off_b); PTR(conv); PTR(conv_w); PTR(ring); PTR(state); PTR(decay);
  VAL(ld_decay); PTR(gate); VAL(ld_gate); PTR(a_exp); PTR(dt_bias); PTR(norm_w); VAL(eps);
  VAL(H); VAL(Hk); VAL(dim); VAL(vdim); VAL(taps); VAL(C); PTR(out);
  PTR(seg_row); PTR(seg_len); PTR(seg_pos); PTR(seg_state); PTR(positions); PTR(row_state);
  VAL(nseg); VAL(rows);
  return a;
}

drtc::GroupedAttnArgs grouped_args(const py::dict& d) {
  const Fields f{d};
  drtc::GroupedAttnArgs a{};
  PTR(out); VAL(ldo); PTR(q); PTR(k); PTR(v); PTR(gate); VAL(ldg); PTR(block_tables);
  VAL(bt_stride); VAL(H); VAL(G); VAL(dimp); VAL(vdimp); VAL(sink); VAL(scale); VAL(cap);
  PTR(q_cu); PTR(start); PTR(tile_seq); PTR(tile_row); VAL(ntiles); VAL(qtile); VAL(nseq);
  PTR(context_lens); PTR(part_ml); PTR(part_o); VAL(B); VAL(per); VAL(nsplits);
  return a;
}

drtc::MemoryArgs memory_args(const py::dict& d) {
  const Fields f{d};
  drtc::MemoryArgs a{};
  PTR(proj); VAL(ldp); VAL(off_k); VAL(off_v); VAL(off_g); VAL(off_i); VAL(off_f); VAL(H); VAL(dim);
  VAL(vdim); VAL(q_scale); VAL(k_scale); PTR(cos_sin); VAL(rot_dims); PTR(log_decay); PTR(i_bias);
  PTR(f_bias); VAL(cap); PTR(norm_w); VAL(silu); VAL(eps); PTR(state); PTR(nrm); PTR(top);
  VAL(slices); PTR(out); VAL(ldo); PTR(seg_row); PTR(seg_len); PTR(seg_pos); PTR(seg_state);
  VAL(nseg); PTR(positions); PTR(row_state); VAL(rows);
  return a;
}

}  // namespace

void bind_hybrid(py::module_& m) {
  m.def("memory_scan", [](int f32, const py::dict& d, int plain, u64 st) {
    return drtc::launch_memory_scan(f32, memory_args(d), plain, S(st));
  });
  m.def("memory_decode", [](int f32, const py::dict& d, u64 st) {
    return drtc::launch_memory_decode(f32, memory_args(d), S(st));
  });
  m.def("side_norm", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::SideNormArgs a{};
    PTR(out); VAL(ldo); PTR(h); PTR(y); VAL(ldy); PTR(yw); PTR(ids); PTR(embed); VAL(embed_scale);
    PTR(w); VAL(W); VAL(eps); VAL(rows);
    return drtc::launch_side_norm(f32, a, S(st));
  });
  m.def("stream_add", [](int f32, u64 out, u64 h, u64 y, int64_t ldy, int rows, int W, u64 st) {
    return drtc::launch_stream_add(f32, P<void>(out), P<float>(h), P<void>(y), ldy, rows, W, S(st));
  });
  m.def("side_gate_gemm", [](u64 out, u64 x, u64 w, u64 embed, int64_t lde, int off, u64 ids, int T,
                             int N, int K, u64 st) {
    return drtc::launch_side_gate_gemm(P<void>(out), P<void>(x), P<void>(w), P<void>(embed), lde, off,
                                       P<const int>(ids), T, N, K, S(st));
  });
  m.def("side_gate", [](int f32, u64 out, u64 z, u64 embed, int64_t lde, int off, u64 ids, int rows,
                        int dim, u64 st) {
    return drtc::launch_side_gate(f32, P<void>(out), P<void>(z), P<void>(embed), lde, off,
                                  P<const int>(ids), rows, dim, S(st));
  });
  m.def("group_rms", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::GroupRmsArgs a{};
    PTR(out); VAL(ldo); PTR(h); PTR(y); VAL(ldy); PTR(s); PTR(ids); PTR(embed); VAL(embed_scale);
    PTR(w); VAL(W); VAL(groups); VAL(eps); VAL(rows);
    return drtc::launch_group_rms(f32, a, S(st));
  });
  m.def("attn_prep", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::AttnPrepArgs a{};
    PTR(proj); VAL(ldp); VAL(off_k); VAL(off_v); VAL(H); VAL(G); VAL(dimp); VAL(vdimp); PTR(conv);
    VAL(taps); PTR(ring); PTR(cos_sin); VAL(rot_dims); PTR(slots); PTR(q); PTR(k); PTR(v);
    PTR(v_first); VAL(vdim); VAL(mix); VAL(lam); PTR(tile_seg); PTR(tile_off); PTR(seg_row); PTR(seg_len);
    PTR(seg_pos); PTR(seg_state); PTR(positions); PTR(row_state); VAL(ntiles); VAL(per);
    return drtc::launch_attn_prep(f32, a, S(st));
  });
  m.def("grouped_any", [](int f32, const py::dict& d, int rows, u64 st) {
    return drtc::launch_grouped_any(f32, grouped_args(d), rows, S(st));
  });
  m.def("grouped_prefill", [](const py::dict& d, u64 st) {
    return drtc::launch_grouped_prefill(grouped_args(d), S(st));
  });
  m.def("grouped_decode", [](const py::dict& d, u64 st) {
    return drtc::launch_grouped_decode(grouped_args(d), S(st));
  });
  m.def("dyt", [](int f32, u64 out, u64 h, u64 y, int ldy, u64 ids, u64 embed, u64 w, u64 b,
                  float alpha, int rows, int W, u64 st) {
    return drtc::launch_dyt(f32, P<void>(out), P<float>(h), P<void>(y), ldy, P<const int>(ids),
                            P<void>(embed), P<float>(w), P<float>(b), alpha, rows, W, S(st));
  });
  m.def("act_glu_f32", [](u64 out, u64 gu, int64_t T, int I, int stride, int act, float limit,
                          u64 st) {
    return drtc::launch_act_glu_f32(P<float>(out), P<float>(gu), T, I, stride, act, limit, S(st));
  });
  m.def("latent_prep", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::LatentPrepArgs a{};
    PTR(proj); VAL(ldp); VAL(off_kv); VAL(H); VAL(dim); VAL(rot); VAL(rot_dims); VAL(R); VAL(LW);
    PTR(norm_w); VAL(eps); PTR(cos_sin); PTR(positions); PTR(slots); PTR(lat); PTR(cache);
    PTR(qa); VAL(rows);
    return drtc::launch_latent_prep(f32, a, S(st));
  });
  m.def("latent_gather", [](u64 out, u64 cache, u64 slots, int rows, int row_bytes, u64 st) {
    return drtc::launch_latent_gather(P<void>(out), P<void>(cache), P<const int64_t>(slots), rows,
                                      row_bytes, S(st));
  });
  m.def("latent_prefill", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::LatentPrefillArgs a{};
    PTR(out); VAL(ldo); PTR(q); VAL(ldq); PTR(kv); VAL(ldkv); VAL(voff); PTR(lat); VAL(LW);
    VAL(R); VAL(H); VAL(dim); VAL(rot); VAL(vdim); PTR(q_cu); PTR(k_cu); PTR(ctx); PTR(tile_seq);
    PTR(tile_q0); VAL(ntiles); VAL(qtile); VAL(nseq); VAL(nq); VAL(window); VAL(scale); PTR(sink);
    PTR(gate); VAL(ldg);
    return drtc::launch_latent_prefill(f32, a, S(st));
  });
  m.def("latent_decode", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::LatentDecodeArgs a{};
    PTR(out); PTR(part_o); PTR(part_ml); PTR(qa); PTR(cache); PTR(block_tables); VAL(bt_stride);
    PTR(context_lens); VAL(B); VAL(H); VAL(R); VAL(LW); VAL(window); VAL(tiles_per_split);
    VAL(nsplits); VAL(scale); PTR(sink); PTR(gate); VAL(ldg);
    return drtc::launch_latent_decode(f32, a, S(st));
  });
  m.def("head_gemm", [](int f32, u64 y, u64 x, u64 w, int B, int H, int N, int K, int64_t yb,
                        int64_t yh, int64_t xb, int64_t xh, u64 st) {
    return drtc::launch_head_gemm(f32, P<void>(y), P<void>(x), P<void>(w), B, H, N, K, yb, yh, xb,
                                  xh, S(st));
  });
  m.def("short_conv", [](int f32, u64 out, u64 proj, int ldp, u64 w, u64 ring, u64 positions,
                         u64 row_off, u64 row_state, int rows, int C, int taps, u64 st) {
    return drtc::launch_short_conv(f32, P<void>(out), P<void>(proj), ldp, P<float>(w),
                                   P<void>(ring), P<const int>(positions), P<const int>(row_off),
                                   P<const int>(row_state), rows, C, taps, S(st));
  });
  m.def("delta_scan", [](int f32, const py::dict& d, int cpl, u64 st) {
    return drtc::launch_delta_scan(f32, delta_args(d), cpl, S(st));
  });
  m.def("delta_decode", [](int f32, const py::dict& d, u64 st) {
    return drtc::launch_delta_decode(f32, delta_args(d), S(st));
  });
  m.def("norm_conv", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::NormConvArgs a{};
    f.ptr("out1", a.out[0]); f.ptr("out2", a.out[1]); PTR(h_out); PTR(h_in); PTR(y); VAL(ldy);
    PTR(ids); PTR(embed); PTR(turns); f.ptr("w1", a.w[0]); f.ptr("w2", a.w[1]);
    f.ptr("b1", a.b[0]); f.ptr("b2", a.b[1]); f.ptr("conv1", a.conv[0]);
    f.ptr("conv2", a.conv[1]); PTR(ring); PTR(tile_seg); PTR(tile_off); PTR(seg_row);
    PTR(seg_len); PTR(seg_pos); PTR(seg_state); PTR(positions); VAL(ntiles); VAL(per); VAL(W);
    VAL(taps); VAL(eps);
    return drtc::launch_norm_conv(f32, a, S(st));
  });
  m.def("relu2", [](int f32, u64 out, int64_t ldo, u64 x, int64_t rows, int cols, u64 st) {
    return drtc::launch_relu2(f32, P<void>(out), ldo, P<void>(x), rows, cols, S(st));
  });
  m.def("softcap", [](int f32, u64 x, int64_t n, float cap, u64 st) {
    return drtc::launch_softcap(f32, P<void>(x), n, cap, S(st));
  });
  m.def("gated_average", [](int f32, const py::dict& d, bool decode, u64 st) {
    const Fields f{d};
    drtc::GatedAverageArgs a{};
    PTR(proj); VAL(ldp); VAL(off_x); VAL(off_g); PTR(zb); PTR(xb); PTR(state); PTR(out); VAL(ldo);
    VAL(C); PTR(seg_row); PTR(seg_len); PTR(seg_pos); PTR(seg_state); VAL(nseg); PTR(chunk_seg);
    PTR(chunk_off); PTR(maps); VAL(nchunks); VAL(chunk); PTR(positions); PTR(row_state); VAL(rows);
    return decode ? drtc::launch_gated_decode(f32, a, S(st)) : drtc::launch_gated_scan(f32, a, S(st));
  });
  m.def("head_prep", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::HeadPrepArgs a{};
    PTR(proj); VAL(ldp); VAL(off_k); VAL(off_v); VAL(H); VAL(G); VAL(dim); VAL(dimp); VAL(vdimp);
    PTR(qb); PTR(kb); PTR(vb); PTR(qn); PTR(kn); VAL(eps); PTR(slots); PTR(q); PTR(k); PTR(v);
    VAL(rows);
    return drtc::launch_head_prep(f32, a, S(st));
  });
  m.def("talk_decode", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::TalkDecodeArgs a{};
    PTR(out); VAL(ldo); PTR(q); PTR(k); PTR(v); PTR(plane); PTR(part_ml); PTR(part_o);
    PTR(block_tables); VAL(bt_stride); PTR(context_lens); PTR(sink); PTR(talk); VAL(scale); VAL(B);
    VAL(H); VAL(G); VAL(dimp); VAL(vdimp); VAL(per); VAL(nsplits);
    return drtc::launch_talk_decode(f32, a, S(st));
  });
  m.def("talk_prefill", [](int f32, const py::dict& d, u64 st) {
    const Fields f{d};
    drtc::TalkPrefillArgs a{};
    PTR(out); VAL(ldo); PTR(q); PTR(k); PTR(v); PTR(stats); PTR(q_cu); PTR(start);
    PTR(block_tables); VAL(bt_stride); PTR(tile_seq); PTR(tile_q0); PTR(stile_seq); PTR(stile_q0);
    VAL(ntiles); VAL(nstiles); VAL(nseq); VAL(nq); PTR(sink); PTR(talk); VAL(scale); VAL(H);
    VAL(G); VAL(dimp); VAL(vdimp); VAL(mfma);
    return drtc::launch_talk_prefill(f32, a, S(st));
  });
}
