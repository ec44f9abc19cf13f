// Bindings shared by the full kernel library (bindings.cpp) and the decoder
// subset (bindings_decoder.cpp): the bf16 / fp32 GEMMs, the sampler, and the
// fp32-residual and paged-attention kernels.
#pragma once
#include <pybind11/pybind11.h>
#include <pybind11/stl.h>
#include <hip/hip_runtime.h>
#include <cstdint>

#include "kernels/api.h"
#include "kernels/residual_api.h"

namespace py = pybind11;
#define P(x) reinterpret_cast<void*>(static_cast<uintptr_t>(x))
#define CP(x) reinterpret_cast<const void*>(static_cast<uintptr_t>(x))
#define FP(x) reinterpret_cast<float*>(static_cast<uintptr_t>(x))
#define CFP(x) reinterpret_cast<const float*>(static_cast<uintptr_t>(x))
#define IP(x) reinterpret_cast<int*>(static_cast<uintptr_t>(x))
#define CIP(x) reinterpret_cast<const int*>(static_cast<uintptr_t>(x))
#define ST(x) reinterpret_cast<hipStream_t>(static_cast<uintptr_t>(x))
typedef uint64_t u64;

inline void bind_decoder(py::module_& m) {
  m.def("gemm_bf16", [](u64 A, int lda, u64 W, int ldw, u64 C, int ldc, u64 bias, u64 R, int ldr, int M, int N,
                        int K, int act, int out_f32, u64 st, u64 wsh, u64 rowstat, u64 colsum, u64 ws,
                        long long ws_bytes) {
    return dnn_gemm_bf16(CP(A), lda, CP(W), ldw, P(C), ldc, CFP(bias), CP(R), ldr, M, N, K, act, out_f32, ST(st),
                         CP(wsh), CFP(rowstat), CFP(colsum), P(ws), ws_bytes);
  }, py::arg("A"), py::arg("lda"), py::arg("W"), py::arg("ldw"), py::arg("C"), py::arg("ldc"), py::arg("bias"),
     py::arg("R"), py::arg("ldr"), py::arg("M"), py::arg("N"), py::arg("K"), py::arg("act"), py::arg("out_f32"),
     py::arg("st"), py::arg("wsh") = 0, py::arg("rowstat") = 0, py::arg("colsum") = 0, py::arg("ws") = 0,
     py::arg("ws_bytes") = 0);
  m.def("sample_topk", [](u64 x, int ld, int M, int N, u64 out, float temperature, int topk, unsigned seed, u64 step,
                          u64 st) {
    return dnn_sample_topk(CP(x), ld, M, N, reinterpret_cast<int*>(out), temperature, topk, seed,
                           reinterpret_cast<const int*>(step), ST(st));
  });
  m.def("argmax_rows", [](u64 x, int ld, int M, int N, u64 out, int f32in, u64 st, u64 out2, u64 pos_inc, u64 part,
                          u64 hist, int hist_ld) {
    return dnn_argmax_rows(CP(x), ld, M, N, IP(out), f32in, ST(st), IP(out2), IP(pos_inc),
                           reinterpret_cast<void*>(static_cast<uintptr_t>(part)), IP(hist), hist_ld);
  }, py::arg("x"), py::arg("ld"), py::arg("M"), py::arg("N"), py::arg("out"), py::arg("f32in"), py::arg("st"),
     py::arg("out2") = 0, py::arg("pos_inc") = 0, py::arg("part") = 0, py::arg("hist") = 0, py::arg("hist_ld") = 0);
  m.def("rows_update", [](u64 x_in, u64 xidx, int xrows, u64 y, u64 yidx, int yrows, int ldy, float mult, u64 y_w,
                          u64 x_out, int ldx, u64 copy, int ldcopy, u64 n_w, u64 h, int ldh, int M, int N, int NP,
                          float eps, int y_f32, int out_f32, u64 st) {
    RowsArgs a;
    a.x_in = CFP(x_in), a.xidx = CIP(xidx), a.y = CP(y), a.yidx = CIP(yidx), a.y_w = CFP(y_w), a.x_out = FP(x_out);
    a.copy = P(copy), a.n_w = CFP(n_w), a.h = P(h), a.xrows = xrows, a.yrows = yrows, a.ldx = ldx, a.ldy = ldy;
    a.ldcopy = ldcopy, a.ldh = ldh, a.M = M, a.N = N, a.NP = NP, a.mult = mult, a.eps = eps;
    return dnn_rows_update(&a, y_f32, out_f32, ST(st));
  });
  m.def("token_gate", [](u64 x, int ldx, u64 w, int ldw, u64 wsh, int K, u64 table, int ldt, int off, u64 tok, int V,
                         u64 g, int ldg, int M, int n, int np, u64 st) {
    return dnn_token_gate(CP(x), ldx, CP(w), ldw, CP(wsh), K, CP(table), ldt, off, CIP(tok), V, P(g), ldg, M, n, np,
                          ST(st));
  });
  m.def("token_gate_f32", [](u64 z, int ldz, u64 table, int ldt, int off, u64 tok, int V, u64 g, int ldg, int M, int n,
                             int np, u64 st) {
    return dnn_token_gate_f32(CFP(z), ldz, CFP(table), ldt, off, CIP(tok), V, FP(g), ldg, M, n, np, ST(st));
  });
  m.def("glu_f32", [](u64 gu, int ldi, u64 out, int ldo, int M, int F, u64 st) {
    return dnn_glu_f32(CFP(gu), ldi, FP(out), ldo, M, F, ST(st));
  });
  m.def("gemm_f32", [](u64 A, int lda, u64 W, int ldw, u64 C, int ldc, u64 bias, int M, int N, int K, u64 st) {
    return dnn_gemm_f32(CFP(A), lda, CFP(W), ldw, FP(C), ldc, CFP(bias), M, N, K, ST(st));
  });
  py::class_<PagedAttnArgs>(m, "PagedAttnArgs")
      .def(py::init([](u64 qkv, int ldq, u64 kp, u64 vp, u64 table, int ldt, int npages, u64 slots, u64 pos, u64 out,
                       int ldo, int M, int H, int G, int DK, int DV, int gate, int window, int keep, float scale) {
        PagedAttnArgs a;
        a.qkv = CP(qkv), a.kp = P(kp), a.vp = P(vp), a.table = CIP(table), a.slots = CIP(slots), a.pos = CIP(pos);
        a.out = P(out), a.ldq = ldq, a.ldo = ldo, a.ldt = ldt, a.npages = npages, a.M = M, a.H = H, a.G = G;
        a.DK = DK, a.DV = DV, a.gate = gate, a.window = window, a.keep = keep, a.scale = scale;
        return a;
      }));
  m.def("paged_write", [](const PagedAttnArgs& a, int f32, u64 st) { return dnn_paged_write(&a, f32, ST(st)); });
  m.def("paged_prefill", [](const PagedAttnArgs& a, u64 tiles, int ntiles, u64 st) {
    return dnn_paged_prefill(&a, CIP(tiles), ntiles, ST(st));
  });
  m.def("paged_decode", [](const PagedAttnArgs& a, u64 rows, int nrows, int splits, u64 ws, long long ws_elems,
                           u64 st) {
    return dnn_paged_decode(&a, CIP(rows), nrows, splits, FP(ws), ws_elems, ST(st));
  });
  m.def("paged_attn_f32", [](const PagedAttnArgs& a, u64 st) { return dnn_paged_attn_f32(&a, ST(st)); });
}
