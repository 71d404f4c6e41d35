// model_registry.hpp -- from a path to a runner.  A GGUF file names its architecture in general.architecture, a model folder in
// config.json; the registry maps the name to what reads the configuration, loads the weights and builds the runner.
#pragma once
#include <functional>

#include "gguf.hpp"
#include "hip_llama.hpp"
#include "hybrid.hpp"

namespace crabml_host {

struct LoadOptions {
  size_t seq_len = 0;    // longest sequence (0: the model's own limit, where its configuration has one)
  bool f32 = false;      // llama: f32 KV cache; hybrid decoder: every activation, product and cache entry f32
  bool use_graph = true;
  size_t pass_rows = 0;  // rows per prompt pass (0: default)
};

inline std::string read_file(const std::string& path) {
  std::ifstream f(path, std::ios::binary);
  if (!f) throw Error(ErrorKind::IOError, "cannot open " + path);
  std::ostringstream s;
  s << f.rdbuf();
  return s.str();
}

// a model folder: config.json + model.safetensors
struct ModelFolder {
  std::string path;
  Json config;
  static bool is_one(const std::string& path) {
    struct stat st;
    return ::stat((path + "/config.json").c_str(), &st) == 0;
  }
  explicit ModelFolder(const std::string& p) : path(p), config(Json::parse(read_file(p + "/config.json"))) {}
  std::string architecture() const { return config.at("architecture").str(); }
};

typedef std::function<std::unique_ptr<ModelRunner>(const ModelFolder&, const HipTensorDeviceRef&, const LoadOptions&)> FolderLoader;
typedef std::function<std::unique_ptr<ModelRunner>(const GGUFFile&, const HipTensorDeviceRef&, const LoadOptions&)> GgufLoader;

// a model class on the hybrid decoder: what reads its config.json, what finds its tensors
inline FolderLoader hybrid_model(HybridConfig (*config)(const Json&), HybridWeights (*weights)(const SafeTensorsFile&, const HybridConfig&, const HipTensorDeviceRef&)) {
  return [config, weights](const ModelFolder& f, const HipTensorDeviceRef& dev, const LoadOptions& o) -> std::unique_ptr<ModelRunner> {
    const HybridConfig c = config(f.config);
    const SafeTensorsFile st(f.path + "/model.safetensors");
    return std::make_unique<HipHybridRunner>(c, weights(st, c, dev), dev, o.seq_len ? o.seq_len : 8192, o.f32, o.use_graph, o.pass_rows);
  };
}
inline const std::map<std::string, FolderLoader>& folder_models() {
  static const std::map<std::string, FolderLoader> m = {
      {"Bifazen", hybrid_model(bifazen_config, bifazen_weights)},
      {"Nilivik", hybrid_model(nilivik_config, nilivik_weights)},
  };
  return m;
}
inline const std::map<std::string, GgufLoader>& gguf_models() {
  static const std::map<std::string, GgufLoader> m = {
      {"llama",
       [](const GGUFFile& g, const HipTensorDeviceRef& dev, const LoadOptions& o) -> std::unique_ptr<ModelRunner> {
         const LlamaConfig c = load_llama_config(g);
         const size_t seq_len = o.seq_len ? o.seq_len : c.seq_len;
         auto r = std::make_unique<HipLlamaRunner>(c, load_llama_weights(g, c, dev), dev, seq_len, !o.f32, o.use_graph, true, 1, 0, nullptr, true, 0, 0, o.pass_rows);
         r->set_seq_cap(seq_len);
         return r;
       }},
  };
  return m;
}

inline std::string model_architecture(const std::string& path) { return ModelFolder::is_one(path) ? ModelFolder(path).architecture() : GGUFFile(path).architecture(); }

inline std::unique_ptr<ModelRunner> load_model(const std::string& path, const HipTensorDeviceRef& dev, const LoadOptions& o) {
  auto unknown = [](const std::string& a) -> Error { return Error(ErrorKind::ModelError, "unsupported architecture " + a); };
  if (ModelFolder::is_one(path)) {
    const ModelFolder f(path);
    auto it = folder_models().find(f.architecture());
    if (it == folder_models().end()) throw unknown(f.architecture());
    return it->second(f, dev, o);
  }
  const GGUFFile g(path);
  auto it = gguf_models().find(g.architecture());
  if (it == gguf_models().end()) throw unknown(g.architecture());
  return it->second(g, dev, o);
}
inline std::vector<std::string> known_architectures() {
  std::vector<std::string> v;
  for (const auto& m : folder_models()) v.push_back(m.first);
  for (const auto& m : gguf_models()) v.push_back(m.first);
  return v;
}

}  // namespace crabml_host
