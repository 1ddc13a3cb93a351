// model_registry.cpp -- config.json + safetensors model folders and the layer-stack model classes.
//
// config.json names the architecture; the registry maps it to the function that reads the rest of the
// configuration into a ti_stack_config and its layers.  Weights come from model.safetensors (an 8-byte
// little-endian header length, a JSON header name -> dtype / shape / data_offsets, the data), widened
// to fp32 tensors in the ModelData as the GGUF reader does with bf16.
#include "model_registry.hpp"

#include <cstring>
#include <filesystem>
#include <fstream>
#include <iterator>
#include <map>
#include <stdexcept>

#include "api_common.hpp"
#include "json.hpp"

namespace turboinfer {
namespace api {

namespace fs = std::filesystem;

namespace {

// One entry of "layers" whose "type" is latent_attention.
void read_latent_attention(const Json& m, ti_stack_layer& L) {
  L.mixer = TI_MIX_LATENT;
  L.heads = m["heads"].integer();
  L.dim = m["dim"].integer();
  L.rot_dim = m["rot_dim"].integer();
  L.vdim = m["vdim"].integer();
  L.q_rank = m["q_rank"].integer();
  L.kv_rank = m["kv_rank"].integer();
  L.scale = (float)m["scale"].number();
  L.rot_base = (float)m["rot"]["base"].number();
  L.rot_dims = m["rot"].has("dims") ? m["rot"]["dims"].integer() : L.rot_dim;
}

// "attention": grouped-query attention with one added to the softmax's denominator.
void read_attention(const Json& m, ti_stack_layer& L) {
  L.mixer = TI_MIX_GQA;
  L.heads = m["heads"].integer();
  L.kv_heads = m["kv_heads"].integer();
  L.dim = m["dim"].integer();
  L.vdim = m["vdim"].integer();
  L.scale = (float)m["scale"].number();
  L.sink_one = 1;
  if (m.has("q_temp") && !m["q_temp"].is_null()) {
    L.temp_coef = (float)m["q_temp"]["coef"].number();
    L.temp_every = (float)m["q_temp"]["every"].number();
    if (!(L.temp_every > 0.0f)) throw std::runtime_error("config.json: q_temp.every must be positive");
  }
  if (m.has("kv_from") && !m["kv_from"].is_null()) {
    L.kv_shared = 1;
    L.kv_from = m["kv_from"].integer();
  }
}

void read_mamba2(const Json& m, ti_stack_layer& L) {
  L.mixer = TI_MIX_SSD;
  L.heads = m["heads"].integer();
  L.vdim = m["vdim"].integer();
  L.state = m["state"].integer();
  L.groups = m["groups"].integer();
  L.norm_groups = m["norm_groups"].integer();
  L.conv = m["conv"].integer();
}

void read_rglru(const Json& m, ti_stack_layer& L) {
  L.mixer = TI_MIX_RGLRU;
  L.mix_width = m["width"].integer();
  L.blocks = m["blocks"].integer();
  L.conv = m["conv"].integer();
}

// The feed-forward of a design whose layers have this kind or none.
void read_mlp(const Json& e, const char* design_kind, ti_stack_layer& L) {
  L.mlp = TI_MLP_NONE;
  if (!e.has("mlp") || e["mlp"].is_null()) return;
  const Json& m = e["mlp"];
  const std::string kind = m["kind"].string();
  if (kind != design_kind) throw std::runtime_error("config.json: feed-forward kind \"" + kind + "\" is not supported");
  if (kind == "dense") {
    L.mlp = TI_MLP_DENSE;
    L.ff = m["ff"].integer();
    return;
  }
  L.mlp = TI_MLP_MOE;
  L.experts = m["router"]["experts"].integer();
  L.top = m["router"]["top"].integer();
  L.ff = m["expert"]["ff"].integer();
}

// Gegepel: latent-attention layers with sandwich layer norms and softmax-routed experts, a range of
// layers looped with shared weights.
StackSpec gegepel_spec(const Json& j) {
  StackSpec s;
  ti_stack_config& c = s.cfg;
  c.vocab = j["vocab"].integer();
  c.width = j["width"].integer();
  c.eps = (float)j["norm"]["eps"].number();
  c.emb_scale = (float)j["embedding"]["scale"].number();
  for (const Json& e : j["layers"].array()) {
    ti_stack_layer L{};
    const std::string type = e["type"].string();
    if (type != "latent_attention") throw std::runtime_error("config.json: layer type \"" + type + "\" is not supported");
    read_latent_attention(e["mixer"], L);
    read_mlp(e, "moe", L);
    s.layers.push_back(L);
  }
  c.layers = (int)s.layers.size();
  if (j.has("loop") && !j["loop"].is_null()) {
    c.loop_start = j["loop"]["start"].integer();
    c.loop_stop = j["loop"]["stop"].integer();
    c.loop_times = j["loop"]["times"].integer();
  }
  return s;
}

// Nogitar: attention, Mamba-2 and RG-LRU layers in any order, RMS norms behind the sublayers only, a bigram
// table and sinusoidal position vectors in the embedding.
StackSpec nogitar_spec(const Json& j) {
  StackSpec s;
  ti_stack_config& c = s.cfg;
  c.vocab = j["vocab"].integer();
  c.width = j["width"].integer();
  c.eps = (float)j["norm"]["eps"].number();
  c.emb_scale = (float)j["embedding"]["scale"].number();
  const Json& b = j["embedding"]["bigram"];
  c.bigram_buckets = b["buckets"].integer();
  c.bigram_mul_prev = b["mul_prev"].integer();
  c.bigram_mul_cur = b["mul_cur"].integer();
  if (c.bigram_buckets < 1) throw std::runtime_error("config.json: bigram.buckets must be positive");
  c.sinusoid = 1;
  c.norm_kind = TI_NORM_RMS;
  c.norm_place = TI_PLACE_POST;
  for (const Json& e : j["layers"].array()) {
    ti_stack_layer L{};
    const std::string type = e["type"].string();
    if (type == "attention") read_attention(e["mixer"], L);
    else if (type == "mamba2") read_mamba2(e["mixer"], L);
    else if (type == "rglru") read_rglru(e["mixer"], L);
    else throw std::runtime_error("config.json: layer type \"" + type + "\" is not supported");
    read_mlp(e, "dense", L);
    s.layers.push_back(L);
  }
  c.layers = (int)s.layers.size();
  return s;
}

const std::map<std::string, StackSpec (*)(const Json&)>& registry() {
  static const std::map<std::string, StackSpec (*)(const Json&)> r = {{"Gegepel", gegepel_spec}, {"Nogitar", nogitar_spec}};
  return r;
}

std::string read_text(const fs::path& p) {
  std::ifstream f(p, std::ios::binary);
  if (!f.is_open()) throw std::runtime_error("cannot open " + p.string());
  return std::string(std::istreambuf_iterator<char>(f), std::istreambuf_iterator<char>());
}

void read_safetensors(const fs::path& path, model::ModelData& out) {
  std::ifstream f(path, std::ios::binary);
  if (!f.is_open()) throw std::runtime_error("cannot open " + path.string());
  const uint64_t size = fs::file_size(path);
  uint64_t hl = 0;
  f.read(reinterpret_cast<char*>(&hl), 8);
  if (!f.good() || hl > size - 8) throw std::runtime_error(path.string() + ": not a safetensors file");
  std::string head(hl, '\0');
  f.read(head.data(), (std::streamsize)hl);
  if (!f.good()) throw std::runtime_error(path.string() + ": short header");
  const uint64_t base = 8 + hl;
  const Json h = Json::parse(head);
  std::vector<uint16_t> half;
  for (const auto& [name, t] : h.object()) {
    if (name == "__metadata__") continue;
    const std::string dt = t["dtype"].string();
    std::vector<size_t> dims;
    size_t n = 1;
    for (const Json& d : t["shape"].array()) {
      dims.push_back((size_t)d.integer());
      n *= dims.back();
    }
    if (dims.empty()) dims.push_back(1);
    const std::vector<Json>& off = t["data_offsets"].array();
    if (off.size() != 2) throw std::runtime_error(path.string() + ": data_offsets of " + name);
    const double b = off[0].number(), e = off[1].number();
    const size_t es = dt == "F32" || dt == "I32" ? 4 : dt == "BF16" || dt == "F16" ? 2 : 0;
    if (!es) throw std::runtime_error(path.string() + ": dtype " + dt + " of " + name + " is not supported");
    if (!(b >= 0 && e >= b && e - b == (double)(n * es) && e <= (double)(size - base)))
      throw std::runtime_error(path.string() + ": extent of " + name);
    f.seekg((std::streamoff)(base + (uint64_t)b));
    core::Tensor v(core::TensorShape(dims), dt == "I32" ? core::DataType::kInt32 : core::DataType::kFloat32);
    if (es == 4) {
      f.read(static_cast<char*>(v.data()), (std::streamsize)(n * 4));
    } else {
      half.resize(n);
      f.read(reinterpret_cast<char*>(half.data()), (std::streamsize)(n * 2));
      float* d = v.data_ptr<float>();
      for (size_t i = 0; i < n; ++i) {
        if (dt == "F16") {
          d[i] = half_to_float(half[i]);
        } else {
          const uint32_t u = (uint32_t)half[i] << 16;
          std::memcpy(d + i, &u, 4);
        }
      }
    }
    if (!f.good()) throw std::runtime_error(path.string() + ": short data for " + name);
    out.add_tensor(name, std::move(v));
  }
}

fs::path model_folder(const std::string& path) {
  const fs::path p(path);
  return fs::is_directory(p) ? p : p.parent_path();
}

}  // namespace

bool is_stack_architecture(const std::string& a) { return registry().count(a) != 0; }

std::vector<std::string> stack_architectures() {
  std::vector<std::string> v;
  for (const auto& kv : registry()) v.push_back(kv.first);
  return v;
}

StackSpec stack_spec(const std::string& text) {
  const Json j = Json::parse(text);
  const std::string a = j["architecture"].string();
  const auto it = registry().find(a);
  if (it == registry().end()) throw std::runtime_error("config.json: architecture \"" + a + "\" is not supported");
  return it->second(j);
}

bool is_model_dir(const std::string& path) {
  std::error_code ec;
  return fs::exists(model_folder(path) / "config.json", ec);
}

model::ModelData load_model_dir(const std::string& path) {
  const fs::path dir = model_folder(path);
  const std::string text = read_text(dir / "config.json");
  const StackSpec s = stack_spec(text);
  model::ModelData m;
  model::ModelMetadata& md = m.metadata();
  md.name = fs::absolute(dir).lexically_normal().filename().string();
  if (md.name.empty()) md.name = "model";
  md.architecture = Json::parse(text)["architecture"].string();
  md.vocab_size = (size_t)s.cfg.vocab;
  md.hidden_size = (size_t)s.cfg.width;
  md.num_layers = s.layers.size();
  for (auto l = s.layers.rbegin(); l != s.layers.rend(); ++l) {   // (the first layer that has the part decides)
    if (l->mixer == TI_MIX_LATENT || l->mixer == TI_MIX_GQA) {
      md.num_heads = (size_t)l->heads;
      md.rope_theta = l->rot_base;
    }
    if (l->mlp != TI_MLP_NONE) md.intermediate_size = (size_t)l->ff;
  }
  md.extra_params["config.json"] = text;
  read_safetensors(fs::is_directory(path) ? dir / "model.safetensors" : fs::path(path), m);
  return m;
}

ti_engine* create_stack_engine(const std::string& config_json, int dtype, int max_seq, int max_batch, int device) {
  StackSpec s = stack_spec(config_json);
  s.cfg.dtype = dtype;
  s.cfg.max_seq = max_seq;
  s.cfg.max_batch = max_batch;
  s.cfg.device = device;
  if (s.layers.empty()) throw std::runtime_error("config.json: no layers");
  ti_engine* e = nullptr;
  check(ti_engine_create_stack(&s.cfg, s.layers.data(), &e), "ti_engine_create_stack");
  return e;
}

ti_engine* build_stack_engine(const model::ModelData& m, int dtype, int max_seq, int max_batch, int device) {
  ti_engine* e = create_stack_engine(m.get_config_param("config.json"), dtype, max_seq, max_batch, device);
  try {
    const int n = ti_engine_weight_count(e);
    for (int i = 0; i < n; ++i) {
      char name[256];
      int rows = 0, cols = 0;
      check(ti_engine_weight_info(e, i, name, sizeof(name), &rows, &cols), "ti_engine_weight_info");
      const core::Tensor* t = m.get_tensor(name);
      if (!t) throw std::runtime_error("the checkpoint lacks tensor " + std::string(name));
      const auto& d = t->shape().dimensions();
      size_t tr = d.empty() ? 0 : d[0];   // rows: every dimension but the last (block-diagonal weights have three)
      for (size_t q = 1; q + 1 < d.size(); ++q) tr *= d[q];
      const size_t tc = d.size() > 1 ? d.back() : 1;
      if (tr != (size_t)rows || tc != (size_t)cols || d.size() > 3)
        throw std::runtime_error("tensor " + std::string(name) + " has the wrong shape (expected " + std::to_string(rows) +
                                 " x " + std::to_string(cols) + ")");
      if (t->dtype() == core::DataType::kFloat32) {
        check(ti_engine_set_weight(e, name, t->data_ptr<float>(), rows, cols), "ti_engine_set_weight");
      } else {
        const std::vector<float> v = to_f32(*t);
        check(ti_engine_set_weight(e, name, v.data(), rows, cols), "ti_engine_set_weight");
      }
    }
  } catch (...) {
    ti_engine_destroy(e);
    throw;
  }
  return e;
}

}  // namespace api
}  // namespace turboinfer

int ti_set_error(int code, const char* fmt, ...);

extern "C" int ti_engine_load(const char* dir, int dtype, int max_seq, int max_batch, int device, ti_engine** out) {
  if (!dir || !out) return ti_set_error(TI_ERR_ARG, "ti_engine_load: null");
  *out = nullptr;
  try {
    *out = turboinfer::api::build_stack_engine(turboinfer::api::load_model_dir(dir), dtype, max_seq, max_batch, device);
  } catch (const std::exception& ex) {
    return ti_set_error(TI_ERR_ARG, "ti_engine_load(%s): %s", dir, ex.what());
  }
  return TI_OK;
}

extern "C" int ti_engine_create_config(const char* config_json, int dtype, int max_seq, int max_batch, int device, ti_engine** out) {
  if (!config_json || !out) return ti_set_error(TI_ERR_ARG, "ti_engine_create_config: null");
  *out = nullptr;
  try {
    *out = turboinfer::api::create_stack_engine(config_json, dtype, max_seq, max_batch, device);
  } catch (const std::exception& ex) {
    return ti_set_error(TI_ERR_ARG, "ti_engine_create_config: %s", ex.what());
  }
  return TI_OK;
}
