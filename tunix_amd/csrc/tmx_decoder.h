// Shared by the translation units that enqueue a decode step.
#pragma once
#include <vector>

#include "tmx_kernels.h"

namespace tmx {

inline size_t align256(size_t v) { return (v + 255) & ~(size_t)255; }

// Optional per-kernel-class timing with HIP events (used by the benchmark only).
struct Prof {
  std::vector<hipEvent_t> ev[TMX_NUM_KERNEL_CLASSES];
  void before(int k, hipStream_t st) { push(k, st); }
  void after(int k, hipStream_t st) { push(k, st); }
  void push(int k, hipStream_t st) {
    hipEvent_t e;
    if (hipEventCreate(&e) != hipSuccess) return;
    (void)hipEventRecord(e, st);
    ev[k].push_back(e);
  }
};

#define TMX_TRY(kind, expr)            \
  {                                    \
    if (prof) prof->before(kind, st);  \
    rc = (expr);                       \
    if (prof) prof->after(kind, st);   \
    if (rc != TMX_OK) return rc;       \
  }

// TMX_FAMILY_DENSE: workspace of a pass of `rows` rows (the first 256 bytes are the status block of every family).
struct DenseWorkspace {
  float* xs;            // residual streams [rows][S][Dp]
  void *xn, *z, *q, *lat, *val, *y, *act;
  int2* place;          // per chunk size of the layers: tmx_row_places of every row (TMX_MIXER_HEADS)
  float* attn_partial;
  float* y_part;        // f32 planes of a projection whose K is split [nsplit][rows][Dp]
  float* logits;        // f32 models: products of the head [rows][Vp]
  void* head_partial;
  size_t total;
};
DenseWorkspace dense_carve(const tmx_model_desc* m, int rows, char* base);
int dense_check(const tmx_model_desc* m);
// Embedding and every layer of one pass; with final_norm w.xn is the head's input afterwards.
int dense_layers(hipStream_t st, const tmx_model_desc* m, const tmx_decode_state* s, const DenseWorkspace& w,
                  int n_seq, int T, bool final_norm, Prof* prof);
inline int pad_to(int v, int k) { return (v + k - 1) / k * k; }

}  // namespace tmx
