// C ABI of the decoder kernels with an fp32 residual and a paged KV cache
// (residual_rows.hip, token_gate.hip, gemm_f32.hip,
// paged_attention.hip).  As in api.h: every
// function enqueues on `st`; 0 = success, negative = rejected shape.
#pragma once
#include <hip/hip_runtime.h>

struct RowsArgs {
  const float* x_in;   // residual rows (nullptr: 0)
  const int* xidx;     // optional gather of x rows (no x_out then), xrows entries exist
  const void* y;       // sublayer output rows (nullptr: none)
  const int* yidx;     // optional gather of y rows
  const float* y_w;    // RMS-norm weight of y (nullptr: y as it is)
  float* x_out;        // updated residual (may be x_in)
  void* copy;          // optional copy of x' as a GEMM operand
  const float* n_w;    // RMS-norm weight of h (nullptr: no h)
  void* h;
  int xrows, yrows, ldx, ldy, ldcopy, ldh, M, N, NP;
  float mult, eps;
};

// One sequence's key range, masks and scales of a paged attention launch.
struct PagedAttnArgs {
  const void* qkv;     // rows [q H*DK | k G*DK | v G*DV | gate H ...], row stride ldq
  void* kp;            // key pages   [page][G][64][DK]
  void* vp;            // value pages [page][G][64][DV]
  const int* table;    // block table: page of (slot, position / 64); < 0: none
  const int* slots;    // per row: block-table row
  const int* pos;      // per row: position of the token
  void* out;           // [row][H*DV], row stride ldo
  int ldq, ldo, ldt, npages, M;
  int H, G, DK, DV;
  int gate;            // first column of the per-head output gate logits in qkv, -1: none
  int window, keep;    // key j seen by query i: j <= i and (i - j < window or j < keep)
  float scale;
};

extern "C" {
int dnn_rows_update(const RowsArgs* a, int y_f32, int out_f32, hipStream_t st);
// g = gelu_tanh(x W^T) * table[tok]: bf16, wsh = W in fragment order; _f32: from z = x W^T
int dnn_token_gate(const void* x, int ldx, const void* w, int ldw, const void* wsh, int K, const void* table, int ldt,
                   int off, const int* tok, int V, void* g, int ldg, int M, int n, int np, hipStream_t st);
int dnn_token_gate_f32(const float* z, int ldz, const float* table, int ldt, int off, const int* tok, int V, float* g,
                       int ldg, int M, int n, int np, hipStream_t st);
int dnn_glu_f32(const float* gu, int ldi, float* out, int ldo, int M, int F, hipStream_t st);
int dnn_gemm_f32(const float* A, int lda, const float* W, int ldw, float* C, int ldc, const float* bias, int M, int N,
                 int K, hipStream_t st);
int dnn_paged_write(const PagedAttnArgs* a, int f32, hipStream_t st);
int dnn_paged_prefill(const PagedAttnArgs* a, const int* tiles, int ntiles, hipStream_t st);
int dnn_paged_decode(const PagedAttnArgs* a, const int* rows, int nrows, int splits, float* ws, long long ws_elems,
                     hipStream_t st);
int dnn_paged_attn_f32(const PagedAttnArgs* a, hipStream_t st);
}
