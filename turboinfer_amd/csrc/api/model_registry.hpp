// model_registry.hpp -- model classes chosen by config.json's "architecture" (not installed).
#pragma once

#include <string>
#include <vector>

#include "ti_engine.h"
#include "turboinfer/model/model_loader.hpp"

namespace turboinfer {
namespace api {

/// A layer-stack model's configuration, as ti_engine_create_stack takes it (dtype / max_seq /
/// max_batch / device left to the caller).
struct StackSpec {
  ti_stack_config cfg{};
  std::vector<ti_stack_layer> layers;
};

bool is_stack_architecture(const std::string& architecture);
std::vector<std::string> stack_architectures();
/// config.json text -> configuration; std::runtime_error naming the key that is missing or wrong.
StackSpec stack_spec(const std::string& config_json);

/// A model folder (config.json + model.safetensors), or a .safetensors file beside its config.json.
model::ModelData load_model_dir(const std::string& path);
bool is_model_dir(const std::string& path);

/// The device engine of a config.json text, weights not set; the caller owns it.
ti_engine* create_stack_engine(const std::string& config_json, int dtype, int max_seq, int max_batch, int device);
/// The device engine of a ModelData whose architecture is registered; the caller owns it.
ti_engine* build_stack_engine(const model::ModelData& m, int dtype, int max_seq, int max_batch, int device);

}  // namespace api
}  // namespace turboinfer
