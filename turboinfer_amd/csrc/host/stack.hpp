// stack.hpp -- layer-stack models inside the decode engine (engine.cpp): configuration, packed
// weights, per-run caches and the launch sequence of a step.  The engine owns the loop around it
// (token feed, graphs, sampling, prefill chunking, slots).
#pragma once

#include <hip/hip_runtime.h>

#include <cstdint>
#include <map>
#include <string>
#include <vector>

#include "ti_engine.h"
#include "ti_stack.h"

namespace ti_host {

struct StackPack {            // one product's fragment-ordered weights
  void* p = nullptr;
  int N = 0, K = 0, kp = 0;
};

struct StackLayer {
  ti_stack_layer c{};
  int dim_p = 0, rot_p = 0, lat_p = 0, vdim_p = 0, na = 0;
  StackPack a, uq, ukt, uk, uv, o, router, gu, down;   // ukt: per head transposed; gu, down: all experts
  float *n1 = nullptr, *n1b = nullptr, *n2 = nullptr, *n2b = nullptr;   // [2][width]: weight, bias
  float *q_norm = nullptr, *c_norm = nullptr, *sink = nullptr;
  const float* rope = nullptr;
  // grouped-query attention (a: [queries | keys | values | gates]), SSD (a: the in projection) and RG-LRU
  // (a: [GELU branch | convolution input], gates: per block, rows (recurrence, input) interleaved)
  int ka = -1, va = -1, ga = 0;            // a's rows of keys, values, gates
  int cin = 0, o0 = 0, bwp = 0, conv_ld = 0;   // convolution channels and its output layout (ti_conv)
  StackPack gates, up;
  float *k_norm = nullptr, *in_b = nullptr, *conv_w = nullptr, *conv_b = nullptr, *dt_bias = nullptr, *a_log = nullptr,
        *d_skip = nullptr, *gate_b = nullptr, *rate = nullptr;
  const float* q_scale = nullptr;          // [position]
};

struct StackRun {             // one pass through one layer
  int layer = 0, pass = -1;   // pass >= 0: the loop entry step comes first
  // per stream slot (slot bytes each): positions' rows, recurrent state, convolution ring
  void* cache = nullptr;      // latent: T [seq_p][lat_p + rot_p]; grouped-query: ti_stack.h blocks (a layer
                              // that shares keys and values points at its source's)
  void* ring = nullptr;       // T [taps][channels]
  float* state = nullptr;
  size_t cache_slot = 0, ring_slot = 0, state_slot = 0;
  bool own_cache = false;
};

// Rows a forward call works on: decode = one row per stream slot, prompt chunk = consecutive positions
// of one slot.
struct StackRows {
  int M = 0;
  const int32_t* pos = nullptr;   // device [M]
  float* h = nullptr;             // device [M][width] residual (embedding rows in, final residual out)
  const float* h0 = nullptr;      // device [M][width] embedding output
  bool chunk = false;
  int slot = 0, pos0 = 0;         // chunk: stream slot and first position (host)
  const int32_t* slots = nullptr; // decode, device [M], nullable: the rows' stream slots (NULL: row m is slot m)
  bool xn_ready = false;          // the embedding's element-type rows are in xn already
  float* layers_out = nullptr;    // host, nullable: residual after every run, run stride layers_stride rows
  size_t layers_stride = 0;
};

struct StackWeight {
  std::string name;
  int rows = 0, cols = 0;
  bool set = false;
};

class StackModel {
 public:
  ti_stack_config c{};
  std::vector<StackLayer> layer;
  std::vector<StackRun> run;
  std::vector<StackWeight> weights;
  size_t weight_bytes = 0, kv_bytes = 0;
  int seq_p = 0, rows_cap = 0, dec_rows = 0;
  void* emb = nullptr;
  float* h0 = nullptr;          // [rows_cap][width]
  void* bigram = nullptr;       // [buckets + 1][width]
  int32_t* hist = nullptr;      // [max_batch][seq_p] tokens by position (with a bigram table)
  float *pe_hi = nullptr, *pe_lo = nullptr;   // sinusoidal position vectors (ti_hip.h ti_step_args)
  int pe_ld = 0;
  void* xn = nullptr;           // T [rows_cap][kpad(width)]: input rows of the next product
  int xn_ld = 0;
  bool recurrent = false;       // some layer carries a state: a slot only goes on where it stands

  ~StackModel();
  static int check(const ti_stack_config& c, const ti_stack_layer* l);
  int create(const ti_stack_config& c, const ti_stack_layer* l, int rows, hipStream_t s);
  int set_weight(const std::string& name, const float* host, int rows, int cols);
  int synth(uint64_t seed, float norm_jitter);
  int fill_kv(int stream, int n, uint64_t seed);
  int ready();                  // every weight set?

  // all runs over `rows`; with `head` the final norm, head product and argmax of every row follow
  int forward(const StackRows& r, bool head, float* logits, unsigned long long* argmax, int32_t* step_ctr, int advance);
  int head(float* h, int M, float* logits, unsigned long long* argmax);
  int fork(int src, int dst, int n);   // copy a slot's cache positions [0, n) and its states

 private:
  hipStream_t s_ = nullptr;
  bool ready_ = false;
  std::vector<void*> allocs_;
  std::map<std::string, int> index_;
  StackPack loop_in_, head_;
  float *loop_step_ = nullptr, *final_norm_ = nullptr;
  // work buffers
  void *cat_ = nullptr, *cq_ = nullptr, *q_ = nullptr, *qa_ = nullptr, *olat_ = nullptr, *attn_ = nullptr,
       *act_ = nullptr, *parts_ = nullptr, *kfrag_ = nullptr, *vfrag_ = nullptr, *part_o_ = nullptr;
  float *a32_ = nullptr, *gate_ = nullptr, *y_ = nullptr, *zr_ = nullptr, *wgt_ = nullptr, *part_ml_ = nullptr, *stage_ = nullptr;
  int32_t *idx_ = nullptr, *list_ = nullptr, *tiles_ = nullptr, *n_tiles_ = nullptr, *map_ = nullptr;
  size_t stage_elems_ = 0, map_elems_ = 0;
  // work buffers of the grouped-query and recurrent mixers
  void *proj_ = nullptr, *conv_ = nullptr;   // T: projections, convolution outputs
  float *dt_ = nullptr, *ys_ = nullptr, *ab_ = nullptr, *gpart_o_ = nullptr, *gpart_ml_ = nullptr;
  std::map<std::pair<float, float>, float*> temps_;

  int alloc(void** p, size_t bytes);
  template <class P>
  int alloc_t(P** p, size_t n) {
    void* v = nullptr;
    const int rc = alloc(&v, n * sizeof(P));
    *p = static_cast<P*>(v);
    return rc;
  }
  int esize() const { return c.dtype == TI_DT_BF16 ? 2 : 4; }
  int kpad(int k) const { return ti_stack_kpad(c.dtype, k); }
  int alloc_pack(StackPack& w, int N, int K, int copies = 1);
  int alloc_layer(StackLayer& L);
  int alloc_work();
  int add_weight(const std::string& name, int rows, int cols);
  int set_device(const std::string& name, const float* dev, int rows, int cols);
  int pack(const StackPack& w, const float* src, int64_t rs, int64_t ks, int rows, const std::vector<int32_t>* map,
           size_t elem_off = 0);
  int dense(const StackPack& w, const void* a, int lda, int M, void* out, int ldo, int epi, ti_dense_args extra);
  int add_mixer_weights(int i);
  int alloc_mixer(StackLayer& L);
  int alloc_run(StackRun& r);
  int alloc_mixer_work();
  int host_copy(const float* dev, size_t n, std::vector<float>& out);
  int set_mixer_weight(StackLayer& L, const std::string& t, const float* d, int rows, int cols, bool& known);
  int gqa(const StackLayer& L, const StackRun& run, const StackRows& r);
  int ssd(const StackLayer& L, const StackRun& run, const StackRows& r);
  int rglru(const StackLayer& L, const StackRun& run, const StackRows& r);
  int dense_mlp(const StackLayer& L, int M);
  int attention(const StackLayer& L, const StackRun& run, const StackRows& r);
  bool fused_router(const StackLayer& L, int M) const;
  int experts(const StackLayer& L, int M);
};

}  // namespace ti_host
