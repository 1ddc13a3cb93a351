// stack_mixers.cpp -- grouped-query attention, SSD and RG-LRU layers and the dense feed-forward of the
// layer-stack models (stack.hpp).
//
// Every mixer reads the rows xn and leaves its output product's fp32 rows in y_:
//   attention  dense [queries | keys | values | gates]; prep (norms, query scale, cache append); attention
//              over the cache's fragments with the gate behind it; output product
//   SSD        dense in projection (step sizes fp32); rows of many slots: convolution and recurrence in one
//              launch; prompt chunks: convolution, block scan; gated norm; output product
//   RG-LRU     dense [GELU branch | convolution input]; rows of many slots: convolution, gate products and
//              the recurrence's step in one launch; prompt chunks: convolution, per-block gate product whose
//              epilogue makes the recurrence's coefficients, scan; output product
#include <algorithm>
#include <cmath>

#include "stack.hpp"
#include "ti_hip.h"

int ti_set_error(int code, const char* fmt, ...);

#define TI_TRY(expr)                 \
  do {                               \
    const int _rc = (expr);          \
    if (_rc != TI_OK) return _rc;    \
  } while (0)

namespace ti_host {

namespace {

inline int up(int v, int u) { return (v + u - 1) / u * u; }
std::string lname(int l, const char* t) { return "l" + std::to_string(l) + "." + t; }

std::vector<int32_t> range(int n, int off, int step = 1) {
  std::vector<int32_t> m(n);
  for (int i = 0; i < n; ++i) m[i] = off + i * step;
  return m;
}

}  // namespace

int StackModel::add_mixer_weights(int i) {
  const ti_stack_layer& k = layer[i].c;
  const int W = c.width, inner = k.heads * k.vdim, cin = layer[i].cin;
  auto add = [&](const char* n, int rows, int cols) { add_weight(lname(i, n), rows, cols); };
  switch (k.mixer) {
    case TI_MIX_GQA:
      add("mix.q", k.heads * k.dim, W);
      add("mix.q.norm", k.heads * k.dim, 1);
      if (!k.kv_shared) {
        add("mix.k", k.kv_heads * k.dim, W);
        add("mix.k.norm", k.kv_heads * k.dim, 1);
        add("mix.v", k.kv_heads * k.vdim, W);
      }
      add("mix.g", inner, W);
      add("mix.o", W, inner);
      return TI_OK;
    case TI_MIX_SSD:
      add("mix.in", inner + cin + k.heads, W);
      add("mix.conv", cin, k.conv);
      add("mix.conv.b", cin, 1);
      add("mix.dt_bias", k.heads, 1);
      add("mix.A_log", k.heads, 1);
      add("mix.D", k.heads, 1);
      add("mix.norm", inner, 1);
      add("mix.o", W, inner);
      return TI_OK;
    default: {
      const int w = k.mix_width, bw = w / k.blocks;
      add("mix.y", w, W);
      add("mix.y.b", w, 1);
      add("mix.x", w, W);
      add("mix.x.b", w, 1);
      add("mix.conv", w, k.conv);
      add("mix.conv.b", w, 1);
      add("mix.ra", w, bw);   // [blocks][bw][bw]
      add("mix.ra.b", k.blocks, bw);
      add("mix.ri", w, bw);
      add("mix.ri.b", k.blocks, bw);
      add("mix.lam", w, 1);
      add("mix.o", W, w);
      return TI_OK;
    }
  }
}

int StackModel::alloc_mixer(StackLayer& L) {
  const ti_stack_layer& k = L.c;
  const int W = c.width, inner = k.heads * k.vdim, kt = c.dtype == TI_DT_BF16 ? 32 : 16;
  switch (k.mixer) {
    case TI_MIX_GQA: {
      L.ga = k.heads * k.dim;
      if (!k.kv_shared) {
        L.ka = L.ga;
        L.va = L.ka + k.kv_heads * k.dim;
        L.ga = L.va + k.kv_heads * k.vdim;
      }
      L.na = L.ga + inner;
      TI_TRY(alloc_pack(L.a, L.na, W));
      TI_TRY(alloc_pack(L.o, W, inner));
      TI_TRY(alloc_t(&L.q_norm, (size_t)k.heads * k.dim));
      TI_TRY(alloc_t(&L.k_norm, (size_t)k.kv_heads * k.dim));
      if (k.sink_one) TI_TRY(alloc_t(&L.sink, (size_t)k.heads));   // (zeros: a score of 0)
      if (k.temp_every > 0.0f) {
        float*& t = temps_[{k.temp_coef, k.temp_every}];
        if (!t) {
          std::vector<float> v(seq_p);
          for (int p = 0; p < seq_p; ++p)
            v[p] = (float)(1.0 + (double)k.temp_coef * std::log(std::floor((p + 1) / (double)k.temp_every) + 1.0));
          TI_TRY(alloc_t(&t, v.size()));
          TI_TRY(ti_memcpy_h2d(t, v.data(), v.size() * 4, s_));
          TI_TRY(ti_stream_sync(s_));
        }
        L.q_scale = t;
      }
      return TI_OK;
    }
    case TI_MIX_SSD:
      recurrent = true;
      L.cin = inner + 2 * k.groups * k.state;
      L.na = inner + L.cin + k.heads;
      L.o0 = up(inner, 16);
      L.bwp = up(k.state, kt);
      L.conv_ld = L.o0 + 2 * k.groups * L.bwp;
      TI_TRY(alloc_pack(L.a, L.na, W));
      TI_TRY(alloc_pack(L.o, W, inner));
      TI_TRY(alloc_t(&L.q_norm, (size_t)inner));
      for (float** p : {&L.dt_bias, &L.a_log, &L.d_skip}) TI_TRY(alloc_t(p, (size_t)k.heads));
      break;
    default:
      recurrent = true;
      L.cin = k.mix_width;
      L.na = 2 * k.mix_width;
      L.bwp = kpad(k.mix_width / k.blocks);
      L.conv_ld = k.blocks * L.bwp;
      TI_TRY(alloc_pack(L.a, L.na, W));
      TI_TRY(alloc_pack(L.o, W, k.mix_width));
      TI_TRY(alloc_pack(L.gates, 2 * (k.mix_width / k.blocks), k.mix_width / k.blocks, k.blocks));
      TI_TRY(alloc_t(&L.in_b, (size_t)L.na));
      TI_TRY(alloc_t(&L.gate_b, (size_t)L.na));
      TI_TRY(alloc_t(&L.rate, (size_t)k.mix_width));
  }
  TI_TRY(alloc_t(&L.conv_w, (size_t)L.cin * k.conv));
  return alloc_t(&L.conv_b, (size_t)L.cin);
}

int StackModel::alloc_run(StackRun& r) {
  const StackLayer& L = layer[r.layer];
  const ti_stack_layer& k = L.c;
  const size_t B = c.max_batch, es = esize();
  if (k.mixer == TI_MIX_LATENT) r.cache_slot = (size_t)seq_p * (L.lat_p + L.rot_p) * es;
  if (k.mixer == TI_MIX_GQA) r.cache_slot = (size_t)k.kv_heads * (seq_p / 64) * ti_gqa_block_elems(c.dtype, k.dim, k.vdim) * es;
  if (L.cin) {
    r.ring_slot = (size_t)k.conv * L.cin * es;
    r.state_slot = k.mixer == TI_MIX_SSD ? (size_t)k.heads * k.vdim * up(k.state, 4) * 4 : (size_t)k.mix_width * 4;
    TI_TRY(alloc(&r.ring, B * r.ring_slot));
    TI_TRY(alloc_t(&r.state, B * r.state_slot / 4));
  }
  if (k.mixer == TI_MIX_GQA && k.kv_shared) {
    r.cache = run[k.kv_from].cache;   // (no loops: run i is layer i)
  } else if (r.cache_slot) {
    r.own_cache = true;
    TI_TRY(alloc(&r.cache, B * r.cache_slot));
    kv_bytes += B * r.cache_slot;
  }
  kv_bytes += B * (r.ring_slot + r.state_slot);
  return TI_OK;
}

int StackModel::alloc_mixer_work() {
  const size_t R = rows_cap, es = esize();
  size_t proj = 0, conv = 0, dt = 0, ys = 0, ab = 0, po = 0, pml = 0;
  for (const auto& L : layer) {
    const ti_stack_layer& k = L.c;
    if (k.mixer == TI_MIX_GQA) {
      for (int M = 1; M <= dec_rows; ++M) {
        const size_t ms = (size_t)M * ti_gqa_splits(M, k.heads, k.kv_heads, c.max_seq) * k.heads;
        po = std::max(po, ms * up(k.vdim, 16));
        pml = std::max(pml, ms * 2);
      }
    } else if (k.mixer != TI_MIX_LATENT) {
      proj = std::max<size_t>(proj, up(L.na, 8));
      conv = std::max<size_t>(conv, L.conv_ld);
      if (k.mixer == TI_MIX_SSD) {
        dt = std::max<size_t>(dt, k.heads);
        ys = std::max<size_t>(ys, up(k.heads * k.vdim, 4));
      } else {
        ab = std::max<size_t>(ab, (size_t)2 * k.mix_width);
      }
    }
  }
  if (po) {
    TI_TRY(alloc_t(&gpart_o_, po));
    TI_TRY(alloc_t(&gpart_ml_, pml));
  }
  if (proj) {
    TI_TRY(alloc(&proj_, R * proj * es));
    TI_TRY(alloc(&conv_, R * conv * es));
  }
  if (dt) {
    TI_TRY(alloc_t(&dt_, R * dt));
    TI_TRY(alloc_t(&ys_, R * ys));
  }
  return ab ? alloc_t(&ab_, R * ab) : TI_OK;
}

// ------------------------------------------------------------------ weights
int StackModel::host_copy(const float* dev, size_t n, std::vector<float>& out) {
  out.resize(n);
  TI_TRY(ti_memcpy_d2h(out.data(), dev, n * 4, s_));
  return ti_stream_sync(s_);
}

int StackModel::set_mixer_weight(StackLayer& L, const std::string& t, const float* d, int rows, int cols, bool& known) {
  const ti_stack_layer& k = L.c;
  const int W = c.width;
  const size_t n = (size_t)rows * cols;
  auto vec = [&](float* dst) -> int { return ti_memcpy_d2d(dst, d, n * 4, s_); };
  auto part = [&](int off) -> int {
    const auto m = range(rows, off);
    return pack(L.a, d, W, 1, rows, &m);
  };
  if (t == "mlp.up" && k.mlp == TI_MLP_DENSE) return pack(L.up, d, W, 1, rows, nullptr);
  if (t == "mlp.down" && k.mlp == TI_MLP_DENSE) return pack(L.down, d, k.ff, 1, rows, nullptr);
  if (k.mixer != TI_MIX_LATENT) {
    if (t == "mix.o") return pack(L.o, d, cols, 1, rows, nullptr);
    if (t == "mix.conv") {   // [channels][taps] -> [taps][channels]
      std::vector<float> v, o(n);
      TI_TRY(host_copy(d, n, v));
      for (int i = 0; i < rows; ++i)
        for (int j = 0; j < cols; ++j) o[(size_t)j * rows + i] = v[(size_t)i * cols + j];
      TI_TRY(ti_memcpy_h2d(L.conv_w, o.data(), n * 4, s_));
      return ti_stream_sync(s_);
    }
    if (t == "mix.conv.b") return vec(L.conv_b);
  }
  if (k.mixer == TI_MIX_GQA) {
    if (t == "mix.q") return part(0);
    if (t == "mix.k") return part(L.ka);
    if (t == "mix.v") return part(L.va);
    if (t == "mix.g") return part(L.ga);
    if (t == "mix.q.norm") return vec(L.q_norm);
    if (t == "mix.k.norm") return vec(L.k_norm);
  } else if (k.mixer == TI_MIX_SSD) {
    if (t == "mix.in") return part(0);
    if (t == "mix.dt_bias") return vec(L.dt_bias);
    if (t == "mix.A_log") return vec(L.a_log);
    if (t == "mix.D") return vec(L.d_skip);
    if (t == "mix.norm") return vec(L.q_norm);
  } else if (k.mixer == TI_MIX_RGLRU) {
    const int w = k.mix_width, bw = w / k.blocks;
    if (t == "mix.y") return part(0);
    if (t == "mix.x") return part(w);
    if (t == "mix.y.b") return vec(L.in_b);
    if (t == "mix.x.b") return vec(L.in_b + w);
    if (t == "mix.ra" || t == "mix.ri") {
      const auto m = range(bw, t == "mix.ri", 2);
      for (int b = 0; b < k.blocks; ++b)
        TI_TRY(pack(L.gates, d + (size_t)b * bw * bw, bw, 1, bw, &m, (size_t)b * up(2 * bw, 16) * L.gates.kp));
      return TI_OK;
    }
    std::vector<float> v, o;
    if (t == "mix.ra.b" || t == "mix.ri.b") {
      TI_TRY(host_copy(d, n, v));
      TI_TRY(host_copy(L.gate_b, 2 * n, o));
      for (size_t i = 0; i < n; ++i) o[2 * i + (t == "mix.ri.b")] = v[i];
      TI_TRY(ti_memcpy_h2d(L.gate_b, o.data(), o.size() * 4, s_));
      return ti_stream_sync(s_);
    }
    if (t == "mix.lam") {
      TI_TRY(host_copy(d, n, v));
      for (float& x : v) x = (float)(8.0 * (x > 0.0f ? x + std::log1p(std::exp(-(double)x)) : std::log1p(std::exp((double)x))));
      TI_TRY(ti_memcpy_h2d(L.rate, v.data(), n * 4, s_));
      return ti_stream_sync(s_);
    }
  }
  known = false;
  return TI_OK;
}

// ------------------------------------------------------------------ forward
int StackModel::gqa(const StackLayer& L, const StackRun& run, const StackRows& r) {
  const ti_stack_layer& k = L.c;
  const int M = r.M, lda = up(L.na, 4), ldo = kpad(k.heads * k.vdim);
  char* cache = static_cast<char*>(run.cache) + (r.chunk ? (size_t)r.slot * run.cache_slot : 0);
  TI_TRY(dense(L.a, xn, kpad(c.width), M, a32_, lda, TI_DE_F32, {}));
  ti_gqa_prep_args p{};
  p.a32 = a32_;
  p.lda = lda;
  p.M = M;
  p.heads = k.heads;
  p.kv_heads = k.kv_heads;
  p.dim = k.dim;
  p.vdim = k.vdim;
  p.k_off = L.ka;
  p.v_off = L.va;
  p.q_w = L.q_norm;
  p.k_w = L.k_norm;
  p.q_scale = L.q_scale;
  p.pos = r.pos;
  p.slot = r.slots;
  p.q = q_;
  p.cache = cache;
  p.slot_stride = r.chunk ? 0 : (int64_t)(run.cache_slot / esize());
  p.seq_p = seq_p;
  p.eps = c.eps;
  p.dtype = c.dtype;
  TI_TRY(ti_gqa_prep(&p, s_));
  ti_gqa_attn_args f{};
  f.q = q_;
  f.cache = cache;
  f.slot_stride = p.slot_stride;
  f.pos = r.pos;
  f.slot = r.slots;
  f.sink = L.sink;
  f.gate = a32_ + L.ga;
  f.out = attn_;
  f.part_o = gpart_o_;
  f.part_ml = gpart_ml_;
  f.scale = k.scale;
  f.M = M;
  f.pos0 = r.pos0;
  f.heads = k.heads;
  f.kv_heads = k.kv_heads;
  f.dim = k.dim;
  f.vdim = k.vdim;
  f.seq_p = seq_p;
  f.ldg = lda;
  f.ldo = ldo;
  f.dtype = c.dtype;
  if (r.chunk && M > 16) {
    TI_TRY(ti_gqa_prefill(&f, s_));
  } else {
    if (M > dec_rows) return ti_set_error(TI_ERR_ARG, "engine: %d decode rows, %d buffered", M, dec_rows);
    f.splits = ti_gqa_splits(M, k.heads, k.kv_heads, c.max_seq);
    TI_TRY(ti_gqa_decode(&f, s_));
  }
  return dense(L.o, attn_, ldo, M, y_, c.width, TI_DE_F32, {});
}

int StackModel::ssd(const StackLayer& L, const StackRun& run, const StackRows& r) {
  const ti_stack_layer& k = L.c;
  const int M = r.M, inner = k.heads * k.vdim, lda = up(L.na, 8), ldy = up(inner, 4), ldo = kpad(inner);
  ti_dense_args da{};
  da.t_cols = L.na - k.heads;
  da.out2 = dt_;
  da.ld2 = k.heads;
  TI_TRY(dense(L.a, xn, kpad(c.width), M, proj_, lda, TI_DE_ACT, da));
  ti_ssd_args s{};
  s.dt = dt_;
  s.dt_bias = L.dt_bias;
  s.a_log = L.a_log;
  s.d = L.d_skip;
  s.state = run.state;
  s.y = ys_;
  s.pos = r.pos;
  s.slot = r.slots;
  s.M = M;
  s.heads = k.heads;
  s.vdim = k.vdim;
  s.state_n = k.state;
  s.groups = k.groups;
  s.taps = k.conv;
  s.ldy = ldy;
  s.slot0 = r.slot;
  s.dtype = c.dtype;
  if (r.chunk) {
    ti_conv_args v{};
    v.x = static_cast<char*>(proj_) + (size_t)inner * esize();
    v.ring = run.ring;
    v.w = L.conv_w;
    v.b = L.conv_b;
    v.out = conv_;
    v.pos = r.pos;
    v.M = M;
    v.channels = L.cin;
    v.taps = k.conv;
    v.act = TI_CONV_SILU;
    v.ldx = lda;
    v.ldo = L.conv_ld;
    v.c0 = inner;
    v.o0 = L.o0;
    v.bw = k.state;
    v.bwp = L.bwp;
    v.slot0 = r.slot;
    v.dtype = c.dtype;
    TI_TRY(ti_conv(&v, s_));
    s.a = conv_;
    s.lda = L.conv_ld;
    s.o0 = L.o0;
    TI_TRY(ti_ssd_scan(&s, s_));
  } else {
    s.a = proj_;
    s.lda = lda;
    s.conv_w = L.conv_w;
    s.conv_b = L.conv_b;
    s.ring = run.ring;
    TI_TRY(ti_ssd_step(&s, s_));
  }
  ti_ssd_norm_args n{};
  n.y = ys_;
  n.raw = proj_;
  n.w = L.q_norm;
  n.out = attn_;
  n.ring = r.chunk ? run.ring : nullptr;
  n.pos = r.pos;
  n.eps = c.eps;
  n.M = M;
  n.inner = inner;
  n.groups = k.norm_groups;
  n.lda = lda;
  n.ldy = ldy;
  n.ldo = ldo;
  n.channels = L.cin;
  n.taps = k.conv;
  n.slot0 = r.slot;
  n.dtype = c.dtype;
  TI_TRY(ti_ssd_norm(&n, s_));
  return dense(L.o, attn_, ldo, M, y_, c.width, TI_DE_F32, {});
}

int StackModel::rglru(const StackLayer& L, const StackRun& run, const StackRows& r) {
  const ti_stack_layer& k = L.c;
  const int M = r.M, w = k.mix_width, bw = w / k.blocks, lda = up(L.na, 8), ldo = kpad(w);
  char* x = static_cast<char*>(proj_) + (size_t)w * esize();
  ti_dense_args da{};
  da.add = L.in_b;
  da.act = TI_ACT_GELU_TANH;
  da.act_cols = w;
  da.t_cols = L.na;
  TI_TRY(dense(L.a, xn, kpad(c.width), M, proj_, lda, TI_DE_ACT, da));
  if (!r.chunk) {
    ti_lru_step_args t{};
    t.x = x;
    t.y = proj_;
    t.ring = run.ring;
    t.conv_w = L.conv_w;
    t.conv_b = L.conv_b;
    t.gates = L.gates.p;
    t.gate_b = L.gate_b;
    t.lru_rate = L.rate;
    t.state = run.state;
    t.out = attn_;
    t.pos = r.pos;
    t.slot = r.slots;
    t.M = M;
    t.channels = w;
    t.blocks = k.blocks;
    t.taps = k.conv;
    t.ldx = lda;
    t.ldo = ldo;
    t.dtype = c.dtype;
    TI_TRY(ti_lru_step(&t, s_));
    return dense(L.o, attn_, ldo, M, y_, c.width, TI_DE_F32, {});
  }
  ti_conv_args v{};
  v.x = x;
  v.ring = run.ring;
  v.w = L.conv_w;
  v.b = L.conv_b;
  v.out = conv_;
  v.pos = r.pos;
  v.M = M;
  v.channels = w;
  v.taps = k.conv;
  v.act = TI_CONV_LINEAR;
  v.ldx = lda;
  v.ldo = L.conv_ld;
  v.bw = bw;
  v.bwp = L.bwp;
  v.slot0 = r.slot;
  v.dtype = c.dtype;
  TI_TRY(ti_conv(&v, s_));
  ti_dense_args g{};
  g.batch = k.blocks;
  g.w_batch = (int64_t)up(2 * bw, 16) * L.gates.kp;
  g.a_batch = L.bwp;
  g.add = L.gate_b;
  g.lru_rate = L.rate;
  TI_TRY(dense(L.gates, conv_, L.conv_ld, M, ab_, 2 * w, TI_DE_LRU, g));
  ti_lru_scan_args s{};
  s.ab = ab_;
  s.y = proj_;
  s.x = x;
  s.out = attn_;
  s.state = run.state;
  s.ring = run.ring;
  s.pos = r.pos;
  s.M = M;
  s.channels = w;
  s.taps = k.conv;
  s.ldy = lda;
  s.ldo = ldo;
  s.slot0 = r.slot;
  s.dtype = c.dtype;
  TI_TRY(ti_lru_scan(&s, s_));
  return dense(L.o, attn_, ldo, M, y_, c.width, TI_DE_F32, {});
}

int StackModel::dense_mlp(const StackLayer& L, int M) {
  const int ldact = kpad(L.c.ff);
  ti_dense_args d{};
  d.act = TI_ACT_GELU_ERF;
  d.act_cols = d.t_cols = L.c.ff;
  TI_TRY(dense(L.up, xn, kpad(c.width), M, act_, ldact, TI_DE_ACT, d));
  return dense(L.down, act_, ldact, M, y_, c.width, TI_DE_F32, {});
}

}  // namespace ti_host
