// stack.cpp -- layer-stack models (stack.hpp): weight layout, caches and the launches of one forward.
//
// A forward is, per run:
//   rownorm   residual += post-norm of the previous sublayer, pre-norm of this one
//             (loop entry: [x ; x0] -> loop.in product + step vector first)
//   dense     one fused projection [query latent | latent | rotated key part | head gates]
//   prep      latent norms, rotary, cache append, gates
//   dense     queries from their latent, rotary in the epilogue
//   attention decode rows: carried into latent space (dense per head, split attention, merge, dense per
//             head with the gate); prompt chunks: keys / values expanded into fragments + chunk attention
//   dense     output projection
//             (grouped-query attention, SSD and RG-LRU layers: stack_mixers.cpp)
//   rownorm   residual += post-norm, pre-norm of the feed-forward
//             (decode-sized row counts: with the router product and the choice of experts)
//   dense     router; route; dense grouped gate/up with SiLU * up; dense grouped down
//             (dense feed-forward: up with GELU, down)
// Models with post-norms only have the element-type copy of the residual in the pre-norms' place.
#include "stack.hpp"

#include <algorithm>
#include <cmath>
#include <cstring>

#include "ti_hip.h"

int ti_set_error(int code, const char* fmt, ...);
int ti_check_hip(hipError_t e, const char* what);

#define S_HIP(expr, what)                                \
  do {                                                   \
    hipError_t _e = (expr);                              \
    if (_e != hipSuccess) return ti_check_hip(_e, what); \
  } while (0)
#define TI_TRY(expr)                 \
  do {                               \
    const int _rc = (expr);          \
    if (_rc != TI_OK) return _rc;    \
  } while (0)

namespace ti_host {

namespace {

inline int up(int v, int u) { return (v + u - 1) / u * u; }

// Source dimension j of a rotated part -> its place: the pairs (i, i + rot_dims / 2) side by side.
// Queries and keys use the same order, so their products are unchanged.
int pair_place(int j, int rot_dims) {
  const int half = rot_dims / 2;
  if (j >= rot_dims) return j;
  return j < half ? 2 * j : 2 * (j - half) + 1;
}

std::string lname(int l, const char* t) { return "l" + std::to_string(l) + "." + t; }

int check_latent(const ti_stack_config& c, const ti_stack_layer& L, int i) {
  if (L.heads < 1 || L.dim < 1 || L.rot_dim < 2 || L.rot_dim % 2 || L.vdim < 1 || L.q_rank < 1 || L.kv_rank < 1 ||
      L.rot_dims < 0 || L.rot_dims > L.rot_dim || L.rot_dims % 2 || !(L.rot_base > 0.0f))
    return ti_set_error(TI_ERR_ARG, "layer %d: latent attention sizes", i);
  const int lim = c.dtype == TI_DT_BF16 ? 2048 : 1024;
  if (L.vdim > 256 || ti_stack_kpad(c.dtype, L.kv_rank) > lim)
    return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: vdim %d (at most 256), kv_rank %d (at most %d)", i, L.vdim, L.kv_rank, lim);
  if (L.q_rank + L.kv_rank + L.rot_dim + L.heads > 15996)
    return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: q_rank + kv_rank + rot_dim + heads > 15996", i);
  return TI_OK;
}

int check_mixer(const ti_stack_config& c, const ti_stack_layer* l, int i) {
  const ti_stack_layer& L = l[i];
  switch (L.mixer) {
    case TI_MIX_LATENT: return check_latent(c, L, i);
    case TI_MIX_GQA:
      if (L.heads < 1 || L.kv_heads < 1 || L.heads % L.kv_heads || L.dim < 1 || L.vdim < 1 || L.temp_every < 0.0f)
        return ti_set_error(TI_ERR_ARG, "layer %d: attention sizes (heads %d, kv_heads %d, dim %d, vdim %d)", i, L.heads,
                            L.kv_heads, L.dim, L.vdim);
      if (L.vdim > 256 || L.dim > 1024 || (L.heads + L.kv_heads) * L.dim > 32768)
        return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: dim %d (at most 1024), vdim %d (at most 256)", i, L.dim, L.vdim);
      if (L.kv_shared) {
        const ti_stack_layer* K = L.kv_from >= 0 && L.kv_from < i ? l + L.kv_from : nullptr;
        if (!K || K->mixer != TI_MIX_GQA || K->kv_shared || K->heads != L.heads || K->kv_heads != L.kv_heads || K->dim != L.dim ||
            K->vdim != L.vdim || c.loop_times > 0)
          return ti_set_error(TI_ERR_ARG, "layer %d: cannot share the keys and values of layer %d", i, L.kv_from);
      }
      return TI_OK;
    case TI_MIX_SSD:
      if (L.heads < 1 || L.vdim < 1 || L.state < 1 || L.groups < 1 || L.heads % L.groups || L.norm_groups < 1 ||
          L.heads * L.vdim % L.norm_groups || L.conv < 1)
        return ti_set_error(TI_ERR_ARG, "layer %d: SSD sizes (heads %d, vdim %d, state %d, groups %d, norm_groups %d, conv %d)", i,
                            L.heads, L.vdim, L.state, L.groups, L.norm_groups, L.conv);
      if (L.state > 256 || L.heads * L.vdim > 32768 || L.conv > 64)
        return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: state %d (at most 256), heads * vdim %d (at most 32768), conv %d (at most 64)",
                            i, L.state, L.heads * L.vdim, L.conv);
      return TI_OK;
    case TI_MIX_RGLRU:
      if (L.mix_width < 1 || L.blocks < 1 || L.mix_width % L.blocks || L.conv < 1)
        return ti_set_error(TI_ERR_ARG, "layer %d: RG-LRU sizes (width %d, blocks %d, conv %d)", i, L.mix_width, L.blocks, L.conv);
      if (L.conv > 64 || L.mix_width / L.blocks > ti_lru_step_max_block(c.dtype))
        return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: conv %d (at most 64), blocks of %d (at most %d)", i, L.conv,
                            L.mix_width / L.blocks, ti_lru_step_max_block(c.dtype));
      return TI_OK;
    default: return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: mixer %d", i, L.mixer);
  }
}

}  // namespace

StackModel::~StackModel() {
  for (void* p : allocs_) hipFree(p);
}

int StackModel::alloc(void** p, size_t bytes) {
  TI_TRY(ti_malloc(p, std::max<size_t>(bytes, 16)));
  allocs_.push_back(*p);
  if (bytes) S_HIP(hipMemsetAsync(*p, 0, bytes, s_), "hipMemsetAsync(alloc)");
  return TI_OK;
}

int StackModel::alloc_pack(StackPack& w, int N, int K, int copies) {
  w.N = N;
  w.K = K;
  w.kp = kpad(K);
  const size_t b = ti_stack_weight_bytes(c.dtype, N, K) * (size_t)copies;
  weight_bytes += b;
  return alloc(&w.p, b);
}

int StackModel::check(const ti_stack_config& c, const ti_stack_layer* l) {
  if (c.vocab < 1 || c.width < 1 || c.layers < 1 || c.max_seq < 1 || c.max_batch < 1 || c.width > 16128)
    return ti_set_error(TI_ERR_ARG, "ti_engine_create_stack: sizes (vocab %d, width %d, layers %d)", c.vocab, c.width, c.layers);
  if (c.dtype != TI_DT_BF16 && c.dtype != TI_DT_F32) return ti_set_error(TI_ERR_ARG, "ti_engine_create_stack: dtype %d", c.dtype);
  if (c.loop_times < 0 || (c.loop_times > 0 && (c.loop_start < 0 || c.loop_stop > c.layers || c.loop_start >= c.loop_stop)))
    return ti_set_error(TI_ERR_ARG, "ti_engine_create_stack: loop [%d, %d) x %d", c.loop_start, c.loop_stop, c.loop_times);
  if ((c.norm_kind != TI_NORM_LAYER && c.norm_kind != TI_NORM_RMS) || (c.norm_place != TI_PLACE_SANDWICH && c.norm_place != TI_PLACE_POST))
    return ti_set_error(TI_ERR_ARG, "ti_engine_create_stack: norm kind %d, place %d", c.norm_kind, c.norm_place);
  if (c.bigram_buckets < 0) return ti_set_error(TI_ERR_ARG, "ti_engine_create_stack: %d bigram buckets", c.bigram_buckets);
  for (int i = 0; i < c.layers; ++i) {
    const ti_stack_layer& L = l[i];
    TI_TRY(check_mixer(c, l, i));
    if (L.mlp == TI_MLP_DENSE && L.ff < 1) return ti_set_error(TI_ERR_ARG, "layer %d: ff %d", i, L.ff);
    if (L.mlp != TI_MLP_NONE && L.mlp != TI_MLP_MOE && L.mlp != TI_MLP_DENSE) return ti_set_error(TI_ERR_UNSUPPORTED, "layer %d: feed-forward %d", i, L.mlp);
    if (L.mlp == TI_MLP_MOE && (L.experts < 1 || L.experts > 1024 || L.top < 1 || L.top > L.experts || L.top > 64 || L.ff < 1))
      return ti_set_error(TI_ERR_ARG, "layer %d: %d experts, top %d, ff %d", i, L.experts, L.top, L.ff);
  }
  return TI_OK;
}

int StackModel::add_weight(const std::string& name, int rows, int cols) {
  index_[name] = (int)weights.size();
  weights.push_back({name, rows, cols, false});
  stage_elems_ = std::max(stage_elems_, (size_t)rows * cols);
  map_elems_ = std::max(map_elems_, (size_t)rows);
  return TI_OK;
}

int StackModel::alloc_layer(StackLayer& L) {
  const ti_stack_layer& k = L.c;
  const int kt = c.dtype == TI_DT_BF16 ? 32 : 16, W = c.width;
  if (k.mixer == TI_MIX_LATENT) {
    L.dim_p = kpad(k.dim);
    L.rot_p = up(k.rot_dim, kt);
    L.lat_p = kpad(k.kv_rank);
    L.vdim_p = up(k.vdim, 16);
    L.na = k.q_rank + k.kv_rank + k.rot_dim + k.heads;
    TI_TRY(alloc_pack(L.a, L.na, W));
    TI_TRY(alloc_pack(L.uq, k.heads * (L.dim_p + L.rot_p), k.q_rank));
    TI_TRY(alloc_pack(L.ukt, L.lat_p, k.dim, k.heads));
    TI_TRY(alloc_pack(L.uk, k.heads * L.dim_p, k.kv_rank));
    TI_TRY(alloc_pack(L.uv, k.heads * L.vdim_p, k.kv_rank));
    TI_TRY(alloc_pack(L.o, W, k.heads * k.vdim));
    TI_TRY(alloc_t(&L.q_norm, (size_t)k.q_rank));
    TI_TRY(alloc_t(&L.c_norm, (size_t)k.kv_rank));
    TI_TRY(alloc_t(&L.sink, (size_t)k.heads));
  } else {
    TI_TRY(alloc_mixer(L));
  }
  for (float** n : {&L.n1, &L.n1b, &L.n2, &L.n2b}) TI_TRY(alloc_t(n, (size_t)2 * W));   // weight, bias
  if (k.mlp == TI_MLP_MOE) {
    TI_TRY(alloc_pack(L.router, k.experts, W));
    TI_TRY(alloc_pack(L.gu, 2 * k.ff, W, k.experts));
    TI_TRY(alloc_pack(L.down, W, k.ff, k.experts));
  } else if (k.mlp == TI_MLP_DENSE) {
    TI_TRY(alloc_pack(L.up, k.ff, W));
    TI_TRY(alloc_pack(L.down, W, k.ff));
  }
  return TI_OK;
}

int StackModel::create(const ti_stack_config& cfg, const ti_stack_layer* l, int rows, hipStream_t s) {
  c = cfg;
  s_ = s;
  seq_p = up(c.max_seq, 128);
  dec_rows = std::max(c.max_batch, 16);
  rows_cap = std::max(rows, dec_rows);
  const int W = c.width;
  layer.resize((size_t)c.layers);
  // rotary tables, shared by layers with the same geometry; the places past rot_dims do not turn
  std::map<std::tuple<int, int, int, float>, float*> tables;
  for (int i = 0; i < c.layers; ++i) {
    StackLayer& L = layer[i];
    L.c = l[i];
    TI_TRY(alloc_layer(L));
    if (L.c.mixer != TI_MIX_LATENT) continue;
    float*& t = tables[std::make_tuple(L.rot_p, L.c.rot_dim, L.c.rot_dims, L.c.rot_base)];
    if (!t) {
      const int pairs = L.rot_p / 2, turn = L.c.rot_dims / 2;
      std::vector<float> cs((size_t)seq_p * pairs * 2);
      for (int p = 0; p < seq_p; ++p)
        for (int j = 0; j < pairs; ++j) {
          const double a = j < turn ? p * std::pow((double)L.c.rot_base, -2.0 * j / L.c.rot_dims) : 0.0;
          cs[((size_t)p * pairs + j) * 2] = (float)std::cos(a);
          cs[((size_t)p * pairs + j) * 2 + 1] = (float)std::sin(a);
        }
      TI_TRY(alloc_t(&t, cs.size()));
      TI_TRY(ti_memcpy_h2d(t, cs.data(), cs.size() * 4, s_));
    }
    L.rope = t;
  }
  // running order
  auto add_run = [&](int i, int pass) { run.push_back({i, pass, nullptr}); };
  const int l0 = c.loop_times > 0 ? c.loop_start : c.layers, l1 = c.loop_times > 0 ? c.loop_stop : c.layers;
  for (int i = 0; i < l0; ++i) add_run(i, -1);
  for (int t = 0; t < c.loop_times; ++t)
    for (int i = l0; i < l1; ++i) add_run(i, i == l0 ? t : -1);
  for (int i = l1; i < c.layers; ++i) add_run(i, -1);
  for (auto& r : run) TI_TRY(alloc_run(r));
  // the checkpoint's tensors
  TI_TRY(alloc(&emb, (size_t)c.vocab * W * esize()));
  weight_bytes += (size_t)c.vocab * W * esize();
  add_weight("embed", c.vocab, W);
  if (c.bigram_buckets > 0) {
    const size_t n = (size_t)(c.bigram_buckets + 1) * W;
    TI_TRY(alloc(&bigram, n * esize()));
    weight_bytes += n * esize();
    TI_TRY(alloc_t(&hist, (size_t)c.max_batch * seq_p));
    add_weight("bigram", c.bigram_buckets + 1, W);
  }
  if (c.sinusoid) {
    pe_ld = up(W, 2);
    const int hi = up(seq_p, 256) / 256;
    std::vector<float> t((size_t)std::max(hi, 256) * pe_ld);
    auto fill = [&](float** dst, int n, int step) -> int {
      for (int p = 0; p < n; ++p)
        for (int e = 0; e < pe_ld; ++e) {
          const double a = (double)p * step * std::pow(10000.0, -2.0 * (e / 2) / W);
          t[(size_t)p * pe_ld + e] = (float)(e % 2 ? std::cos(a) : std::sin(a));
        }
      TI_TRY(alloc_t(dst, (size_t)n * pe_ld));
      TI_TRY(ti_memcpy_h2d(*dst, t.data(), (size_t)n * pe_ld * 4, s_));
      return ti_stream_sync(s_);
    };
    TI_TRY(fill(&pe_hi, hi, 256));
    TI_TRY(fill(&pe_lo, 256, 1));
  }
  if (c.loop_times > 0) {
    add_weight("loop.in", W, 2 * W);
    add_weight("loop.step", c.loop_times, W);
    TI_TRY(alloc_pack(loop_in_, W, 2 * W));
    TI_TRY(alloc_t(&loop_step_, (size_t)c.loop_times * W));
  }
  for (int i = 0; i < c.layers; ++i) {
    const ti_stack_layer& k = layer[i].c;
    for (const char* n : {"norm1", "norm1b", "norm2", "norm2b"}) {
      if ((n[4] == '2' && k.mlp == TI_MLP_NONE) || (n[5] && c.norm_place == TI_PLACE_POST)) continue;
      add_weight(lname(i, n), W, 1);
      if (c.norm_kind == TI_NORM_LAYER) add_weight(lname(i, n) + ".b", W, 1);
    }
    if (k.mixer == TI_MIX_LATENT) {
      add_weight(lname(i, "mix.dq"), k.q_rank, W);
      add_weight(lname(i, "mix.dq.norm"), k.q_rank, 1);
      add_weight(lname(i, "mix.uq"), k.heads * (k.dim + k.rot_dim), k.q_rank);
      add_weight(lname(i, "mix.dkv"), k.kv_rank + k.rot_dim, W);
      add_weight(lname(i, "mix.dkv.norm"), k.kv_rank, 1);
      add_weight(lname(i, "mix.uk"), k.heads * k.dim, k.kv_rank);
      add_weight(lname(i, "mix.uv"), k.heads * k.vdim, k.kv_rank);
      add_weight(lname(i, "mix.sink"), k.heads, 1);
      add_weight(lname(i, "mix.g"), k.heads, W);
      add_weight(lname(i, "mix.o"), W, k.heads * k.vdim);
    } else {
      TI_TRY(add_mixer_weights(i));
    }
    if (k.mlp == TI_MLP_DENSE) {
      add_weight(lname(i, "mlp.up"), k.ff, W);
      add_weight(lname(i, "mlp.down"), W, k.ff);
    }
    if (k.mlp != TI_MLP_MOE) continue;
    add_weight(lname(i, "mlp.router"), k.experts, W);
    for (int e = 0; e < k.experts; ++e) {
      const std::string p = lname(i, "mlp.e") + std::to_string(e);
      add_weight(p + ".gate", k.ff, W);
      add_weight(p + ".up", k.ff, W);
      add_weight(p + ".down", W, k.ff);
    }
  }
  add_weight("final.norm", W, 1);
  if (c.norm_kind == TI_NORM_LAYER) add_weight("final.norm.b", W, 1);
  add_weight("head", c.vocab, W);
  TI_TRY(alloc_t(&final_norm_, (size_t)2 * W));
  TI_TRY(alloc_pack(head_, c.vocab, W));
  TI_TRY(alloc_t(&stage_, stage_elems_));
  TI_TRY(alloc_t(&map_, map_elems_));
  return alloc_work();
}

int StackModel::alloc_work() {
  const size_t R = rows_cap, es = esize();
  const int W = c.width;
  size_t cq = 0, q = 0, qa = 0, at = 0, a32 = 0, hd = 0, E = 1, n = 0, act = 0, kf = 0, vf = 0, po = 0, pml = 0, tiles = 1;
  for (const auto& L : layer) {
    const ti_stack_layer& k = L.c;
    if (k.mlp == TI_MLP_DENSE) act = std::max(act, R * kpad(k.ff));
    if (k.mixer == TI_MIX_LATENT) {
      cq = std::max<size_t>(cq, kpad(k.q_rank));
      q = std::max<size_t>(q, (size_t)k.heads * (L.dim_p + L.rot_p));
      qa = std::max<size_t>(qa, (size_t)k.heads * L.lat_p);
      at = std::max<size_t>(at, kpad(k.heads * k.vdim));
      a32 = std::max<size_t>(a32, up(L.na, 4));
      hd = std::max<size_t>(hd, k.heads);
      kf = std::max<size_t>(kf, (size_t)k.heads * seq_p * L.dim_p);
      vf = std::max<size_t>(vf, (size_t)k.heads * seq_p * L.vdim_p);
      for (int M = 1; M <= dec_rows; ++M) {
        const size_t ms = (size_t)M * ti_latent_attn_splits(M, k.heads, c.max_seq) * k.heads;
        po = std::max(po, ms * L.lat_p);
        pml = std::max(pml, ms * 2);
      }
    } else {
      at = std::max<size_t>(at, kpad(k.mixer == TI_MIX_RGLRU ? k.mix_width : k.heads * k.vdim));
      if (k.mixer == TI_MIX_GQA) {
        q = std::max<size_t>(q, (size_t)k.heads * up(k.dim, 32));
        a32 = std::max<size_t>(a32, up(L.na, 4));
      }
    }
    if (k.mlp == TI_MLP_MOE) {
      E = std::max<size_t>(E, k.experts);
      n = std::max(n, R * k.top);
      act = std::max(act, R * k.top * kpad(k.ff));
      for (int t : {16, 64})
        tiles = std::max<size_t>(tiles, ti_route_max_tiles(t == 16 ? std::min<int>(64, R) : (int)R, k.experts, k.top, t));
      tiles = std::max<size_t>(tiles, (size_t)8 * k.top);
    }
  }
  xn_ld = kpad(W);
  TI_TRY(alloc(&xn, R * xn_ld * es));
  TI_TRY(alloc(&cq_, R * cq * es));
  TI_TRY(alloc(&q_, R * q * es));
  TI_TRY(alloc(&qa_, (size_t)dec_rows * qa * es));
  TI_TRY(alloc(&olat_, (size_t)dec_rows * qa * es));
  TI_TRY(alloc(&attn_, R * at * es));
  TI_TRY(alloc(&kfrag_, kf * es));
  TI_TRY(alloc(&vfrag_, vf * es));
  TI_TRY(alloc(&part_o_, po * es));
  TI_TRY(alloc_t(&part_ml_, pml));
  TI_TRY(alloc_t(&a32_, R * a32));
  TI_TRY(alloc_t(&gate_, R * hd));
  TI_TRY(alloc_t(&y_, R * W));
  TI_TRY(alloc_t(&h0, R * W));
  if (c.loop_times > 0) TI_TRY(alloc(&cat_, R * kpad(2 * W) * es));
  if (act) TI_TRY(alloc(&act_, act * es));
  if (n) {
    TI_TRY(alloc(&parts_, n * W * es));
    TI_TRY(alloc_t(&zr_, R * E));
    TI_TRY(alloc_t(&wgt_, n));
    TI_TRY(alloc_t(&idx_, n));
    TI_TRY(alloc_t(&list_, n));
    TI_TRY(alloc_t(&tiles_, tiles * 4));
    TI_TRY(alloc_t(&n_tiles_, (size_t)1));
  }
  return alloc_mixer_work();
}

// ------------------------------------------------------------------ weights
int StackModel::pack(const StackPack& w, const float* src, int64_t rs, int64_t ks, int rows, const std::vector<int32_t>* map,
                     size_t elem_off) {
  if (map) TI_TRY(ti_memcpy_h2d(map_, map->data(), map->size() * 4, s_));
  TI_TRY(ti_stack_pack(src, rs, ks, rows, w.K, map ? map_ : nullptr, c.dtype, static_cast<char*>(w.p) + elem_off * esize(), s_));
  return map ? ti_stream_sync(s_) : TI_OK;   // (the map buffer is reused)
}

int StackModel::set_device(const std::string& name, const float* d, int rows, int cols) {
  const auto it = index_.find(name);
  if (it == index_.end()) return ti_set_error(TI_ERR_ARG, "set_weight: the model has no tensor %s", name.c_str());
  StackWeight& wt = weights[it->second];
  if (wt.rows != rows || wt.cols != cols)
    return ti_set_error(TI_ERR_ARG, "set_weight: %s is %d x %d, expected %d x %d", name.c_str(), rows, cols, wt.rows, wt.cols);
  const int W = c.width;
  auto vec = [&](float* dst) -> int { return ti_memcpy_d2d(dst, d, (size_t)rows * cols * 4, s_); };
  auto range = [&](int n, int off) {
    std::vector<int32_t> m(n);
    for (int i = 0; i < n; ++i) m[i] = off + i;
    return m;
  };
  wt.set = true;
  if (name == "embed") return ti_stack_convert(d, (uint64_t)rows * cols, c.dtype, emb, s_);
  if (name == "head") return pack(head_, d, W, 1, rows, nullptr);
  if (name == "bigram") return ti_stack_convert(d, (uint64_t)rows * cols, c.dtype, bigram, s_);
  if (name == "loop.in") return pack(loop_in_, d, 2 * W, 1, rows, nullptr);
  if (name == "loop.step") return vec(loop_step_);
  if (name == "final.norm") return vec(final_norm_);
  if (name == "final.norm.b") return vec(final_norm_ + W);
  const size_t dot = name.find('.');
  StackLayer& L = layer[(size_t)std::atoi(name.c_str() + 1)];
  const ti_stack_layer& k = L.c;
  const std::string t = name.substr(dot + 1);
  const std::pair<const char*, float*> norms[] = {{"norm1", L.n1}, {"norm1b", L.n1b}, {"norm2", L.n2}, {"norm2b", L.n2b}};
  for (const auto& n : norms) {
    if (t == n.first) return vec(n.second);
    if (t == std::string(n.first) + ".b") return vec(n.second + W);
  }
  if (k.mixer != TI_MIX_LATENT || k.mlp == TI_MLP_DENSE) {
    bool known = true;
    TI_TRY(set_mixer_weight(L, t, d, rows, cols, known));
    if (known) return TI_OK;
  }
  if (t == "mix.dq") {
    const auto m = range(rows, 0);
    return pack(L.a, d, W, 1, rows, &m);
  }
  if (t == "mix.dkv") {
    auto m = range(rows, k.q_rank);
    for (int j = 0; j < k.rot_dim; ++j) m[k.kv_rank + j] = k.q_rank + k.kv_rank + pair_place(j, k.rot_dims);
    return pack(L.a, d, W, 1, rows, &m);
  }
  if (t == "mix.g") {
    const auto m = range(rows, k.q_rank + k.kv_rank + k.rot_dim);
    return pack(L.a, d, W, 1, rows, &m);
  }
  if (t == "mix.dq.norm") return vec(L.q_norm);
  if (t == "mix.dkv.norm") return vec(L.c_norm);
  if (t == "mix.sink") return vec(L.sink);
  if (t == "mix.uq") {
    std::vector<int32_t> m(rows);
    for (int r = 0; r < rows; ++r) {
      const int h = r / (k.dim + k.rot_dim), j = r % (k.dim + k.rot_dim);
      m[r] = h * (L.dim_p + L.rot_p) + (j < k.dim ? j : L.dim_p + pair_place(j - k.dim, k.rot_dims));
    }
    return pack(L.uq, d, k.q_rank, 1, rows, &m);
  }
  if (t == "mix.uk") {
    std::vector<int32_t> m(rows);
    for (int r = 0; r < rows; ++r) m[r] = r / k.dim * L.dim_p + r % k.dim;
    TI_TRY(pack(L.uk, d, k.kv_rank, 1, rows, &m));
    for (int h = 0; h < k.heads; ++h)   // transposed, per head: row = latent element, k = head dimension
      TI_TRY(pack(L.ukt, d + (size_t)h * k.dim * k.kv_rank, 1, k.kv_rank, k.kv_rank, nullptr, (size_t)h * L.lat_p * L.ukt.kp));
    return TI_OK;
  }
  if (t == "mix.uv") {
    std::vector<int32_t> m(rows);
    for (int r = 0; r < rows; ++r) m[r] = r / k.vdim * L.vdim_p + r % k.vdim;
    return pack(L.uv, d, k.kv_rank, 1, rows, &m);
  }
  if (t == "mix.o") return pack(L.o, d, cols, 1, rows, nullptr);
  if (t == "mlp.router") return pack(L.router, d, W, 1, rows, nullptr);
  if (t.compare(0, 5, "mlp.e") == 0) {
    const int e = std::atoi(t.c_str() + 5);
    const std::string p = t.substr(t.rfind('.') + 1);
    if (p == "down") return pack(L.down, d, k.ff, 1, rows, nullptr, (size_t)e * up(W, 16) * L.down.kp);
    std::vector<int32_t> m(rows);
    for (int r = 0; r < rows; ++r) m[r] = 2 * r + (p == "up");
    return pack(L.gu, d, W, 1, rows, &m, (size_t)e * up(2 * k.ff, 16) * L.gu.kp);
  }
  return ti_set_error(TI_ERR_ARG, "set_weight: %s", name.c_str());
}

int StackModel::set_weight(const std::string& name, const float* host, int rows, int cols) {
  if (!host || rows < 1 || cols < 1 || (size_t)rows * cols > stage_elems_)
    return ti_set_error(TI_ERR_ARG, "set_weight: %s is %d x %d", name.c_str(), rows, cols);
  TI_TRY(ti_memcpy_h2d(stage_, host, (size_t)rows * cols * 4, s_));
  TI_TRY(set_device(name, stage_, rows, cols));
  return ti_stream_sync(s_);
}

int StackModel::ready() {
  if (ready_) return TI_OK;
  for (const auto& w : weights)
    if (!w.set) return ti_set_error(TI_ERR_ARG, "engine: weight %s has not been set", w.name.c_str());
  ready_ = true;
  return TI_OK;
}

// Random weights of the configuration: norms 1 (+- jitter), biases and sinks 0, products scaled so that
// unit-variance inputs give unit-variance outputs.
int StackModel::synth(uint64_t seed, float jitter) {
  for (size_t i = 0; i < weights.size(); ++i) {
    const StackWeight w = weights[i];
    const bool vecw = w.cols == 1, bias = w.name.size() > 2 && w.name.compare(w.name.size() - 2, 2, ".b") == 0;
    const bool sink = w.name.size() > 5 && w.name.compare(w.name.size() - 5, 5, ".sink") == 0;
    const float scale = vecw ? jitter : w.name == "embed" ? 1.7320508f : w.name == "loop.step" ? 0.1f : std::sqrt(3.0f / (float)w.cols);
    TI_TRY(ti_fill_uniform_f32(seed, (uint32_t)(1000 + i), (uint64_t)w.rows * w.cols, scale, vecw && !bias && !sink ? 1.0f : 0.0f,
                               stage_, s_));
    TI_TRY(set_device(w.name, stage_, w.rows, w.cols));
  }
  return ti_stream_sync(s_);
}

int StackModel::fill_kv(int stream, int n, uint64_t seed) {
  uint32_t tid = 0x200000u;
  for (auto& r : run) {
    const StackLayer& L = layer[r.layer];
    const size_t es = esize();
    char* cache = static_cast<char*>(r.cache) + (size_t)stream * r.cache_slot;
    if (r.own_cache && L.c.mixer == TI_MIX_LATENT) {
      TI_TRY(ti_stack_fill(seed, tid++, (uint64_t)n * (r.cache_slot / seq_p / es), 1.0f, c.dtype, cache, s_));
    } else if (r.own_cache) {
      const size_t head = r.cache_slot / L.c.kv_heads, used = head / seq_p * up(n, 64);
      for (int h = 0; h < L.c.kv_heads; ++h) TI_TRY(ti_stack_fill(seed, tid++, used / es, 1.0f, c.dtype, cache + h * head, s_));
    }
    if (r.ring)
      TI_TRY(ti_stack_fill(seed, tid++, r.ring_slot / es, 1.0f, c.dtype, static_cast<char*>(r.ring) + (size_t)stream * r.ring_slot, s_));
    if (r.state)
      TI_TRY(ti_stack_fill(seed, tid++, r.state_slot / 4, 1.0f, TI_DT_F32, r.state + (size_t)stream * (r.state_slot / 4), s_));
  }
  if (hist) TI_TRY(ti_memset(hist + (size_t)stream * seq_p, 0, (size_t)seq_p * 4, s_));
  return ti_stream_sync(s_);
}

int StackModel::fork(int src, int dst, int n) {
  if (src == dst) return TI_OK;
  auto copy = [&](void* base, size_t slot, size_t off, size_t bytes) -> int {
    char* b = static_cast<char*>(base);
    return ti_memcpy_d2d(b + (size_t)dst * slot + off, b + (size_t)src * slot + off, bytes, s_);
  };
  for (auto& r : run) {
    const StackLayer& L = layer[r.layer];
    if (r.own_cache && L.c.mixer == TI_MIX_LATENT) {
      TI_TRY(copy(r.cache, r.cache_slot, 0, r.cache_slot / seq_p * n));
    } else if (r.own_cache) {
      const size_t head = r.cache_slot / L.c.kv_heads;
      for (int h = 0; h < L.c.kv_heads; ++h) TI_TRY(copy(r.cache, r.cache_slot, h * head, head / seq_p * up(n, 64)));
    }
    if (r.ring) TI_TRY(copy(r.ring, r.ring_slot, 0, r.ring_slot));
    if (r.state) TI_TRY(copy(r.state, r.state_slot, 0, r.state_slot));
  }
  return hist ? copy(hist, (size_t)seq_p * 4, 0, (size_t)n * 4) : TI_OK;
}

// ------------------------------------------------------------------ forward
int StackModel::dense(const StackPack& w, const void* a, int lda, int M, void* out, int ldo, int epi, ti_dense_args d) {
  d.w = w.p;
  d.a = a;
  d.lda = lda;
  d.M = M;
  if (!d.N) d.N = w.N;
  d.K = w.kp;
  d.out = out;
  d.ldo = ldo;
  d.epi = epi;
  d.dtype = c.dtype;
  if (!d.batch) d.batch = 1;
  return ti_dense(&d, s_);
}

int StackModel::attention(const StackLayer& L, const StackRun& run, const StackRows& r) {
  const ti_stack_layer& k = L.c;
  const int M = r.M, lda32 = up(L.na, 4), cw = L.lat_p + L.rot_p, hw = L.dim_p + L.rot_p, ldq = kpad(k.q_rank);
  const int ldat = kpad(k.heads * k.vdim);
  char* cache = static_cast<char*>(run.cache) + (r.chunk ? (size_t)r.slot * seq_p * cw * esize() : 0);
  const int64_t stride = r.chunk ? 0 : (int64_t)seq_p * cw;
  TI_TRY(dense(L.a, xn, kpad(c.width), M, a32_, lda32, TI_DE_F32, {}));
  ti_latent_prep_args p{};
  p.a32 = a32_;
  p.lda = lda32;
  p.M = M;
  p.q_rank = k.q_rank;
  p.kv_rank = k.kv_rank;
  p.rot_dim = k.rot_dim;
  p.heads = k.heads;
  p.lat_off = k.q_rank;
  p.rot_off = k.q_rank + k.kv_rank;
  p.gate_off = p.rot_off + k.rot_dim;
  p.q_w = L.q_norm;
  p.c_w = L.c_norm;
  p.rope_cs = L.rope;
  p.pos = r.pos;
  p.cq = cq_;
  p.ldq = ldq;
  p.cache = cache;
  p.slot_stride = stride;
  p.lat_p = L.lat_p;
  p.rot_p = L.rot_p;
  p.gate = gate_;
  p.eps = c.eps;
  p.dtype = c.dtype;
  p.slot = r.slots;
  TI_TRY(ti_latent_prep(&p, s_));
  ti_dense_args dq{};
  dq.rope_cs = L.rope;
  dq.pos = r.pos;
  dq.head_w = hw;
  dq.rot_off = L.dim_p;
  TI_TRY(dense(L.uq, cq_, ldq, M, q_, k.heads * hw, TI_DE_ROPE, dq));
  if (r.chunk && M > 16) {
    const int keys = r.pos0 + M;
    ti_dense_args de{};
    de.key_blocks = seq_p / 16;
    de.head_w = L.dim_p;
    TI_TRY(dense(L.uk, cache, cw, keys, kfrag_, 0, TI_DE_KFRAG, de));
    de.head_w = L.vdim_p;
    TI_TRY(dense(L.uv, cache, cw, keys, vfrag_, 0, TI_DE_VFRAG, de));
    ti_latent_prefill_args f{};
    f.q = q_;
    f.kfrag = kfrag_;
    f.vfrag = vfrag_;
    f.cache = cache;
    f.sink = L.sink;
    f.gate = gate_;
    f.out = attn_;
    f.scale = k.scale;
    f.M = M;
    f.pos0 = r.pos0;
    f.heads = k.heads;
    f.dim_p = L.dim_p;
    f.rot_p = L.rot_p;
    f.lat_p = L.lat_p;
    f.vdim = k.vdim;
    f.vdim_p = L.vdim_p;
    f.key_blocks = seq_p / 16;
    f.ldo = ldat;
    f.dtype = c.dtype;
    TI_TRY(ti_latent_attn_prefill(&f, s_));
  } else {
    if (M > dec_rows) return ti_set_error(TI_ERR_ARG, "engine: %d decode rows, %d buffered", M, dec_rows);
    ti_dense_args du{};
    du.batch = k.heads;
    du.w_batch = (int64_t)L.lat_p * L.ukt.kp;
    du.a_batch = hw;
    du.o_batch = L.lat_p;
    TI_TRY(dense(L.ukt, q_, k.heads * hw, M, qa_, k.heads * L.lat_p, TI_DE_T, du));
    ti_latent_attn_args f{};
    f.qa = qa_;
    f.q = q_;
    f.ldqr = hw;
    f.qr_off = L.dim_p;
    f.cache = cache;
    f.slot_stride = stride;
    f.pos = r.pos;
    f.sink = L.sink;
    f.scale = k.scale;
    f.out = olat_;
    f.part_o = part_o_;
    f.part_ml = part_ml_;
    f.M = M;
    f.heads = k.heads;
    f.lat_p = L.lat_p;
    f.rot_p = L.rot_p;
    f.splits = ti_latent_attn_splits(M, k.heads, c.max_seq);
    f.seq_p = seq_p;
    f.dtype = c.dtype;
    f.slot = r.slots;
    if (f.splits > 1) {
      f.out = nullptr;
      TI_TRY(ti_latent_attn_decode(&f, s_));
      ti_latent_out_args u{};
      u.part_o = part_o_;
      u.part_ml = part_ml_;
      u.sink = L.sink;
      u.w = L.uv.p;
      u.w_batch = (int64_t)L.vdim_p * L.uv.kp;
      u.gate = gate_;
      u.out = attn_;
      u.ldo = ldat;
      u.M = M;
      u.heads = k.heads;
      u.lat_p = L.lat_p;
      u.vdim = k.vdim;
      u.splits = f.splits;
      u.dtype = c.dtype;
      TI_TRY(ti_latent_attn_out(&u, s_));
    } else {
      TI_TRY(ti_latent_attn_decode(&f, s_));
      ti_dense_args dv{};
      dv.batch = k.heads;
      dv.N = k.vdim;
      dv.w_batch = (int64_t)L.vdim_p * L.uv.kp;
      dv.a_batch = L.lat_p;
      dv.gate = gate_;
      dv.gate_ld = k.heads;
      TI_TRY(dense(L.uv, olat_, k.heads * L.lat_p, M, attn_, ldat, TI_DE_GATE, dv));
    }
  }
  return dense(L.o, attn_, ldat, M, y_, c.width, TI_DE_F32, {});
}

// Decode-sized row counts route inside the feed-forward's pre-norm launch.
bool StackModel::fused_router(const StackLayer& L, int M) const {
  return c.norm_place == TI_PLACE_SANDWICH && M <= 64 && ti_rownorm_routes(c.width, L.c.experts);
}

int StackModel::experts(const StackLayer& L, int M) {
  const ti_stack_layer& k = L.c;
  const int W = c.width, ldx = kpad(W), ldact = kpad(k.ff);
  const bool routed = fused_router(L, M);   // idx_ / wgt_ written by the norm's launch
  if (!routed) TI_TRY(dense(L.router, xn, ldx, M, zr_, k.experts, TI_DE_F32, {}));
  ti_route_args ra{};
  ra.logits = routed ? nullptr : zr_;
  ra.ld = k.experts;
  ra.M = M;
  ra.E = k.experts;
  ra.top = k.top;
  ra.idx = idx_;
  ra.wgt = wgt_;
  ra.list = list_;
  ra.tiles = tiles_;
  ra.n_tiles = n_tiles_;
  ti_dense_args g{};
  g.w_batch = (int64_t)up(2 * k.ff, 16) * L.gu.kp;
  g.row_div = k.top;
  // few rows: every (row, choice) entry is a tile of its own (an expert two rows share is read twice)
  const bool direct = M == 1 || (long)M * k.top * 2 <= k.experts;
  if (direct) {
    g.tile_rows = 1;
    g.max_tiles = M * k.top;
    g.tiles = idx_;
    if (!routed) TI_TRY(ti_route(&ra, s_));
  } else {
    ra.tile_rows = M <= 64 ? 16 : (long)M * k.top >= 96L * k.experts ? 128 : 64;
    TI_TRY(ti_route(&ra, s_));
    g.tile_rows = ra.tile_rows;
    g.max_tiles = ti_route_max_tiles(M, k.experts, k.top, ra.tile_rows);
    g.tiles = tiles_;
    g.n_tiles = n_tiles_;
    g.rows_in = list_;
  }
  TI_TRY(dense(L.gu, xn, ldx, M, act_, ldact, TI_DE_SWIGLU, g));
  g.rows_in = nullptr;
  g.row_div = 1;
  if (!direct) g.rows_out = list_;
  g.w_batch = (int64_t)up(W, 16) * L.down.kp;
  return dense(L.down, act_, ldact, M, parts_, W, TI_DE_T, g);
}

int StackModel::forward(const StackRows& r, bool with_head, float* logits, unsigned long long* argmax, int32_t* step_ctr,
                        int advance) {
  const int W = c.width, M = r.M;
  if (M < 1 || M > rows_cap) return ti_set_error(TI_ERR_ARG, "engine: %d rows, %d buffered", M, rows_cap);
  // the sublayer output not yet added to the residual: attention rows (y_) or expert outputs
  const float* post = nullptr;
  bool parts = false;
  int top = 0;
  // pre: weights of the norm in front of the next product, NULL with `copy`: its input is the residual
  auto rownorm = [&](const float* pre, void* cat, const StackLayer* route = nullptr, bool copy = false) -> int {
    if (!post && !pre && !cat && !copy) return TI_OK;
    ti_rownorm_args n{};
    n.x = r.h;
    if (post) {
      if (parts) {
        n.parts = parts_;
        n.part_w = wgt_;
        n.top = top;
      } else {
        n.y = y_;
      }
      n.ldy = W;
      n.post_w = post;
      n.post_b = post + W;
    }
    if (pre || copy) {
      n.w = pre;
      n.b = pre ? pre + W : nullptr;
      n.xn = xn;
      n.ldn = kpad(W);
    }
    if (cat) {
      n.cat = cat;
      n.x0 = r.h0;
      n.ldc = kpad(2 * W);
    }
    n.eps = c.eps;
    n.M = M;
    n.H = W;
    n.kind = c.norm_kind;
    n.dtype = c.dtype;
    if (route) {
      n.route_w = route->router.p;
      n.route_idx = idx_;
      n.route_wgt = wgt_;
      n.route_e = route->c.experts;
      n.route_top = route->c.top;
    }
    post = nullptr;
    return ti_rownorm(&n, s_);
  };
  for (size_t i = 0; i < run.size(); ++i) {
    const StackLayer& L = layer[run[i].layer];
    if (run[i].pass >= 0) {
      TI_TRY(rownorm(nullptr, cat_));
      ti_dense_args d{};
      d.add = loop_step_ + (size_t)run[i].pass * W;
      TI_TRY(dense(loop_in_, cat_, kpad(2 * W), M, r.h, W, TI_DE_F32, d));
    }
    const bool sandwich = c.norm_place == TI_PLACE_SANDWICH;
    if (sandwich || i || !r.xn_ready) TI_TRY(rownorm(sandwich ? L.n1 : nullptr, nullptr, nullptr, !sandwich));
    switch (L.c.mixer) {
      case TI_MIX_GQA: TI_TRY(gqa(L, run[i], r)); break;
      case TI_MIX_SSD: TI_TRY(ssd(L, run[i], r)); break;
      case TI_MIX_RGLRU: TI_TRY(rglru(L, run[i], r)); break;
      default: TI_TRY(attention(L, run[i], r));
    }
    post = sandwich ? L.n1b : L.n1;
    parts = false;
    if (L.c.mlp != TI_MLP_NONE) {
      const bool moe = L.c.mlp == TI_MLP_MOE;
      TI_TRY(rownorm(sandwich ? L.n2 : nullptr, nullptr, moe && fused_router(L, M) ? &L : nullptr, !sandwich));
      if (moe) TI_TRY(experts(L, M));
      else TI_TRY(dense_mlp(L, M));
      post = sandwich ? L.n2b : L.n2;
      parts = moe;
      top = L.c.top;
    }
    if (r.layers_out) {
      TI_TRY(rownorm(nullptr, nullptr));
      TI_TRY(ti_memcpy_d2h(r.layers_out + i * r.layers_stride * W, r.h, (size_t)M * W * 4, s_));
    }
  }
  if (!with_head) return rownorm(nullptr, nullptr);
  TI_TRY(rownorm(final_norm_, nullptr));
  ti_dense_args d{};
  d.argmax = argmax;
  d.step_ctr = step_ctr;
  d.advance = advance;
  return dense(head_, xn, kpad(W), M, logits, c.vocab, TI_DE_LOGITS, d);
}

int StackModel::head(float* h, int M, float* logits, unsigned long long* argmax) {
  const int W = c.width;
  ti_rownorm_args n{};
  n.x = h;
  n.w = final_norm_;
  n.b = final_norm_ + W;
  n.xn = xn;
  n.ldn = kpad(W);
  n.eps = c.eps;
  n.M = M;
  n.H = W;
  n.kind = c.norm_kind;
  n.dtype = c.dtype;
  TI_TRY(ti_rownorm(&n, s_));
  ti_dense_args d{};
  d.argmax = argmax;
  return dense(head_, xn, kpad(W), M, logits, c.vocab, TI_DE_LOGITS, d);
}

}  // namespace ti_host
