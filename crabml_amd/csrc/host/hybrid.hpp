// hybrid.hpp -- models on the hybrid decoder (crabml_hip_hybrid_*): configuration (config.json), weights (safetensors), and the
// runner: sequences, batched steps, greedy generation of many prompts.  The Nilivik and Bifazen designs are model classes built on it.
#pragma once
#include <algorithm>
#include <deque>
#include <fstream>
#include <sstream>

#include "model_runner.hpp"
#include "safetensors.hpp"

namespace crabml_host {

struct HybridLayerConfig {
  struct Attention {
    size_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, chunk = 0, window = 0;
    size_t latent = 0, rot = 0;  // latent attention: rank of the latent, rotated key part
    double scale = 0, out_scale = 1, rot_base = 0;
    bool v_mix = false;
  } attn;
  struct Linear {
    size_t heads = 0, dim = 0, vdim = 0;
    std::vector<double> decay;
    double out_scale = 1;
  } lin;
  size_t ff = 0;
};
enum class NormGain { Single, Vector, VectorAroundZero };

struct HybridConfig {
  std::string architecture;
  size_t width = 0, vocab_size = 0;
  double embed_scale = 1, norm_eps = 0, logit_softcap = 0;
  size_t loop_start = 0, loop_stop = 0, loop_times = 0;
  size_t streams = 0;        // residual streams; 0: a plain residual sum
  double position_base = 0;  // of the position vectors added to the embedding; 0: none
  NormGain gain = NormGain::Single;
  std::vector<HybridLayerConfig> layers;
};

// the tensors of a layer as the C ABI takes them; absent ones stay empty
struct HybridLayerWeights {
  HipTensor norm1, norm2, attn_q, attn_k, attn_v, attn_gate, attn_o, attn_bias_amp, attn_bias_rate, attn_sink;
  HipTensor lin_q, lin_k, lin_v, lin_gate, lin_o, lin_norm, ff_up, ff_down, ff_act, ff_gate;
  HipTensor attn_q_bias, attn_k_bias, attn_v_bias, attn_o_bias, attn_q_norm, attn_k_norm, attn_vmix;
  HipTensor attn_latent_down, attn_latent_norm, attn_key_up, attn_value_up;
  HipTensor hc1_in, hc1_out, hc1_mix, hc2_in, hc2_out, hc2_mix;
};
struct HybridWeights {
  HipTensor embed, loop_step, final_norm, head;
  std::vector<HybridLayerWeights> layers;
};

// ---- Nilivik: config.json and tensor names -----------------------------------------------------------------------------------------
inline HybridConfig nilivik_config(const Json& j) {
  HybridConfig c;
  c.architecture = j.at("architecture").str();
  c.width = j.at("width").size();
  c.vocab_size = j.at("vocab").size();
  c.embed_scale = j.at("embedding").at("scale").number();
  c.position_base = 10000.0;
  c.norm_eps = j.at("norm").at("eps").number();
  if (!j["logit_softcap"].is_null()) c.logit_softcap = j["logit_softcap"].number();
  if (!j["loop"].is_null()) {
    c.loop_start = j["loop"].at("start").size();
    c.loop_stop = j["loop"].at("stop").size();
    c.loop_times = j["loop"].at("times").size();
  }
  for (const Json& l : j.at("layers").items()) {
    if (l.at("type").str() != "parallel") throw Error(ErrorKind::NotImplemented, "unknown mixer `" + l.at("type").str() + "`");
    const Json &m = l.at("mixer"), &a = m.at("left"), &r = m.at("right");
    HybridLayerConfig L;
    L.attn.heads = a.at("heads").size();
    L.attn.kv_heads = a.at("kv_heads").size();
    L.attn.dim = a.at("dim").size();
    L.attn.vdim = a.at("vdim").size();
    L.attn.chunk = a.at("mask").at("size").size();
    L.attn.scale = a.at("scale").number();
    L.attn.out_scale = m.at("left_scale").number();
    L.lin.heads = r.at("heads").size();
    L.lin.dim = r.at("dim").size();
    L.lin.vdim = r.at("vdim").size();
    for (const Json& d : r.at("decay").items()) L.lin.decay.push_back(d.number());
    L.lin.out_scale = m.at("right_scale").number();
    if (L.lin.decay.size() != L.lin.heads) throw Error(ErrorKind::ModelError, "`decay` needs one number per head");
    if (!L.attn.heads || !L.lin.heads || !L.attn.chunk) throw Error(ErrorKind::ModelError, "a `parallel` mixer needs heads on both sides and a chunk size");
    if (!l["mlp"].is_null()) {
      if (l["mlp"].at("kind").str() != "dense") throw Error(ErrorKind::NotImplemented, "unknown feed-forward `" + l["mlp"].at("kind").str() + "`");
      L.ff = l["mlp"].at("ff").size();
    }
    c.layers.push_back(std::move(L));
  }
  return c;
}

inline HybridWeights nilivik_weights(const SafeTensorsFile& f, const HybridConfig& c, const HipTensorDeviceRef& dev) {
  HybridWeights w;
  const size_t W = c.width;
  w.embed = f.load("embed", {c.vocab_size, W}, dev);
  w.head = f.load("head", {c.vocab_size, W}, dev);
  w.final_norm = f.load("final.norm", {}, dev);
  if (c.loop_times) w.loop_step = f.load("loop.step", {c.loop_times, W}, dev);
  for (size_t i = 0; i < c.layers.size(); i++) {
    const HybridLayerConfig& L = c.layers[i];
    const std::string p = "l" + std::to_string(i) + ".", a = p + "mix.left.", r = p + "mix.right.", m = p + "mlp.";
    const size_t H = L.attn.heads, G = L.attn.kv_heads, R = L.lin.heads;
    HybridLayerWeights x;
    x.norm1 = f.load(p + "norm1", {}, dev);
    x.attn_q = f.load(a + "q", {H * L.attn.dim, W}, dev);
    x.attn_k = f.load(a + "k", {G * L.attn.dim, W}, dev);
    x.attn_v = f.load(a + "v", {G * L.attn.vdim, W}, dev);
    x.attn_gate = f.load(a + "g", {H * L.attn.vdim, W}, dev);
    x.attn_o = f.load(a + "o", {W, H * L.attn.vdim}, dev);
    x.attn_bias_amp = f.load(a + "r1", {H}, dev);
    x.attn_bias_rate = f.load(a + "r2", {H}, dev);
    x.attn_sink = f.load(a + "sink", {H}, dev);
    x.lin_q = f.load(r + "q", {R * L.lin.dim, W}, dev);
    x.lin_k = f.load(r + "k", {R * L.lin.dim, W}, dev);
    x.lin_v = f.load(r + "v", {R * L.lin.vdim, W}, dev);
    x.lin_gate = f.load(r + "g", {R * L.lin.vdim, W}, dev);
    x.lin_o = f.load(r + "o", {W, R * L.lin.vdim}, dev);
    x.lin_norm = f.load(r + "norm", {R * L.lin.vdim}, dev);
    if (L.ff) {
      x.norm2 = f.load(p + "norm2", {}, dev);
      x.ff_up = f.load(m + "up", {L.ff, W}, dev);
      x.ff_down = f.load(m + "down", {W, L.ff}, dev);
      x.ff_act = f.load(m + "act", {2}, dev);
    }
    w.layers.push_back(std::move(x));
  }
  return w;
}

// ---- Bifazen: config.json and tensor names -----------------------------------------------------------------------------------------
inline HybridConfig bifazen_config(const Json& j) {
  HybridConfig c;
  c.architecture = j.at("architecture").str();
  c.width = j.at("width").size();
  c.vocab_size = j.at("vocab").size();
  c.norm_eps = j.at("norm").at("eps").number();
  c.gain = NormGain::VectorAroundZero;
  c.streams = j.at("streams").size();
  if (!c.streams) throw Error(ErrorKind::ModelError, "`streams` must be at least 1");
  for (const Json& l : j.at("layers").items()) {
    const std::string& type = l.at("type").str();
    const Json& m = l.at("mixer");
    HybridLayerConfig L;
    HybridLayerConfig::Attention& a = L.attn;
    a.heads = m.at("heads").size();
    a.dim = m.at("dim").size();
    a.vdim = m.at("vdim").size();
    a.window = m.at("mask").at("size").size();
    a.scale = m.at("scale").number();
    if (type == "latent_attention") {
      a.latent = m.at("kv_rank").size();
      a.rot = m.at("rot_dim").size();
      a.rot_base = m.at("rot").at("base").number();
      if (m.at("rot").at("dims").size() != a.rot) throw Error(ErrorKind::ModelError, "`rot.dims` must be `rot_dim`: the shared key part is rotated whole");
      if (!a.latent || a.rot % 2) throw Error(ErrorKind::ModelError, "a `latent_attention` mixer needs a latent, and pairs of rotated dimensions");
    } else if (type == "attention") {
      a.kv_heads = m.at("kv_heads").size();
      a.v_mix = !m["v_mix"].is_null() && m["v_mix"].truth();
      if (!a.kv_heads) throw Error(ErrorKind::ModelError, "an `attention` mixer needs key/value heads");
    } else {
      throw Error(ErrorKind::NotImplemented, "unknown mixer `" + type + "`");
    }
    if (!a.heads || !a.window) throw Error(ErrorKind::ModelError, "a mixer needs heads and a window size");
    if (!l["mlp"].is_null()) {
      if (l["mlp"].at("kind").str() != "dense") throw Error(ErrorKind::NotImplemented, "unknown feed-forward `" + l["mlp"].at("kind").str() + "`");
      L.ff = l["mlp"].at("ff").size();
    }
    c.layers.push_back(std::move(L));
  }
  return c;
}

inline HybridWeights bifazen_weights(const SafeTensorsFile& f, const HybridConfig& c, const HipTensorDeviceRef& dev) {
  HybridWeights w;
  const size_t W = c.width, S = c.streams;
  w.embed = f.load("embed", {c.vocab_size, W}, dev);
  w.final_norm = f.load("final.norm", {W}, dev);
  for (size_t i = 0; i < c.layers.size(); i++) {
    const HybridLayerConfig& L = c.layers[i];
    const HybridLayerConfig::Attention& a = L.attn;
    const std::string p = "l" + std::to_string(i) + ".", x = p + "mix.", m = p + "mlp.";
    const size_t H = a.heads, G = a.kv_heads;
    HybridLayerWeights o;
    o.norm1 = f.load(p + "norm1", {W}, dev);
    o.hc1_in = f.load(p + "hc1.in", {S}, dev);
    o.hc1_out = f.load(p + "hc1.out", {S}, dev);
    o.hc1_mix = f.load(p + "hc1.mix", {S, S}, dev);
    o.attn_o = f.load(x + "o", {W, H * a.vdim}, dev);
    if (a.latent) {
      o.attn_q = f.load(x + "q", {H * (a.dim + a.rot), W}, dev);
      o.attn_latent_down = f.load(x + "dkv", {a.latent + a.rot, W}, dev);
      o.attn_latent_norm = f.load(x + "dkv.norm", {a.latent}, dev);
      o.attn_key_up = f.load(x + "uk", {H * a.dim, a.latent}, dev);
      o.attn_value_up = f.load(x + "uv", {H * a.vdim, a.latent}, dev);
    } else {
      o.attn_q = f.load(x + "q", {H * a.dim, W}, dev);
      o.attn_k = f.load(x + "k", {G * a.dim, W}, dev);
      o.attn_v = f.load(x + "v", {G * a.vdim, W}, dev);
      o.attn_q_bias = f.load(x + "q.b", {H * a.dim}, dev);
      o.attn_k_bias = f.load(x + "k.b", {G * a.dim}, dev);
      o.attn_v_bias = f.load(x + "v.b", {G * a.vdim}, dev);
      o.attn_o_bias = f.load(x + "o.b", {W}, dev);
      o.attn_q_norm = f.load(x + "q.norm", {H * a.dim}, dev);
      o.attn_k_norm = f.load(x + "k.norm", {G * a.dim}, dev);
      o.attn_gate = f.load(x + "g", {H, W}, dev);
      if (a.v_mix) o.attn_vmix = f.load(x + "vmix", {}, dev);
    }
    if (L.ff) {
      o.norm2 = f.load(p + "norm2", {W}, dev);
      o.hc2_in = f.load(p + "hc2.in", {S}, dev);
      o.hc2_out = f.load(p + "hc2.out", {S}, dev);
      o.hc2_mix = f.load(p + "hc2.mix", {S, S}, dev);
      o.ff_gate = f.load(m + "gate", {L.ff, W}, dev);
      o.ff_up = f.load(m + "up", {L.ff, W}, dev);
      o.ff_down = f.load(m + "down", {W, L.ff}, dev);
    }
    w.layers.push_back(std::move(o));
  }
  return w;
}

// one sequence's part of a step
struct StepEntry {
  size_t seq = 0;
  std::vector<uint32_t> tokens;
  std::vector<uint32_t> want;  // places among `tokens` whose logits are returned
};

class HipHybridRunner : public ModelRunner {
 public:
  static constexpr size_t STEP_ROWS = 16;  // sequences one decode step takes (crabml_hip_hybrid_decode_greedy)

  HipHybridRunner(HybridConfig conf, const HybridWeights& w, HipTensorDeviceRef device, size_t seq_len, bool f32, bool use_graph = true, size_t pass_rows = 0)
      : conf_(std::move(conf)), device_(std::move(device)), seq_len_(seq_len) {
    crabml_hip_hybrid_config_t c{};
    c.width = conf_.width;
    c.vocab_size = conf_.vocab_size;
    c.n_layers = conf_.layers.size();
    c.loop_start = conf_.loop_start;
    c.loop_stop = conf_.loop_stop;
    c.loop_times = conf_.loop_times;
    c.seq_len = seq_len;
    c.pass_rows = pass_rows;
    c.embed_scale = (float)conf_.embed_scale;
    c.norm_eps = (float)conf_.norm_eps;
    c.logit_softcap = (float)conf_.logit_softcap;
    c.compute = f32 ? CRABML_HIP_F32 : CRABML_HIP_BF16;
    c.flags = (use_graph ? 0 : CRABML_HIP_HYBRID_NO_GRAPH) | (conf_.gain != NormGain::Single ? CRABML_HIP_HYBRID_NORM_VECTOR : 0) |
              (conf_.gain == NormGain::VectorAroundZero ? CRABML_HIP_HYBRID_NORM_ONE_PLUS : 0);
    c.streams = conf_.streams;
    c.position_base = conf_.position_base;
    if (w.layers.size() != conf_.layers.size()) throw Error(ErrorKind::ModelError, "weights do not have n_layers entries");
    std::vector<crabml_hip_hybrid_layer_t> ls(conf_.layers.size());
    for (size_t i = 0; i < ls.size(); i++) {
      const HybridLayerConfig& L = conf_.layers[i];
      const HybridLayerWeights& x = w.layers[i];
      crabml_hip_hybrid_layer_t& o = ls[i];
      o.attn_heads = L.attn.heads;
      o.attn_kv_heads = L.attn.kv_heads;
      o.attn_dim = L.attn.dim;
      o.attn_vdim = L.attn.vdim;
      o.attn_chunk = L.attn.chunk;
      o.attn_score_scale = (float)L.attn.scale;
      o.attn_out_scale = (float)L.attn.out_scale;
      o.lin_heads = L.lin.heads;
      o.lin_dim = L.lin.dim;
      o.lin_vdim = L.lin.vdim;
      o.lin_out_scale = (float)L.lin.out_scale;
      o.lin_decay = L.lin.decay.data();
      o.ff = L.ff;
      o.norm1 = x.norm1.raw();
      o.attn_q = x.attn_q.raw();
      o.attn_k = x.attn_k.raw();
      o.attn_v = x.attn_v.raw();
      o.attn_gate = x.attn_gate.raw();
      o.attn_o = x.attn_o.raw();
      o.attn_bias_amp = x.attn_bias_amp.raw();
      o.attn_bias_rate = x.attn_bias_rate.raw();
      o.attn_sink = x.attn_sink.raw();
      o.lin_q = x.lin_q.raw();
      o.lin_k = x.lin_k.raw();
      o.lin_v = x.lin_v.raw();
      o.lin_gate = x.lin_gate.raw();
      o.lin_o = x.lin_o.raw();
      o.lin_norm = x.lin_norm.raw();
      o.norm2 = x.norm2.raw();
      o.ff_up = x.ff_up.raw();
      o.ff_down = x.ff_down.raw();
      o.ff_act = x.ff_act.raw();
      o.attn_window = L.attn.window;
      o.attn_latent = L.attn.latent;
      o.attn_rot = L.attn.rot;
      o.attn_rot_base = L.attn.rot_base;
      o.attn_q_bias = x.attn_q_bias.raw();
      o.attn_k_bias = x.attn_k_bias.raw();
      o.attn_v_bias = x.attn_v_bias.raw();
      o.attn_o_bias = x.attn_o_bias.raw();
      o.attn_q_norm = x.attn_q_norm.raw();
      o.attn_k_norm = x.attn_k_norm.raw();
      o.attn_vmix = x.attn_vmix.raw();
      o.attn_latent_down = x.attn_latent_down.raw();
      o.attn_latent_norm = x.attn_latent_norm.raw();
      o.attn_key_up = x.attn_key_up.raw();
      o.attn_value_up = x.attn_value_up.raw();
      o.ff_gate = x.ff_gate.raw();
      o.hc1_in = x.hc1_in.raw();
      o.hc1_out = x.hc1_out.raw();
      o.hc1_mix = x.hc1_mix.raw();
      o.hc2_in = x.hc2_in.raw();
      o.hc2_out = x.hc2_out.raw();
      o.hc2_mix = x.hc2_mix.raw();
    }
    crabml_hip_hybrid_weights_t cw{};
    cw.embed = w.embed.raw();
    cw.loop_step = w.loop_step.raw();
    cw.final_norm = w.final_norm.raw();
    cw.head = w.head.raw();
    device_->check(crabml_hip_hybrid_create(device_->raw(), &c, ls.data(), &cw, &ctx_));
  }
  ~HipHybridRunner() override {
    if (ctx_) crabml_hip_hybrid_destroy(ctx_);
  }
  HipHybridRunner(const HipHybridRunner&) = delete;
  HipHybridRunner& operator=(const HipHybridRunner&) = delete;

  const HybridConfig& conf() const { return conf_; }
  size_t slab_bytes() const { return crabml_hip_hybrid_slab_bytes(ctx_); }

  // ---- sequences and batched steps
  size_t open() {
    size_t s = 0;
    device_->check(crabml_hip_hybrid_open(ctx_, &s));
    return s;
  }
  void close(size_t seq) { device_->check(crabml_hip_hybrid_close(ctx_, seq)); }
  size_t length(size_t seq) const { return crabml_hip_hybrid_len(ctx_, seq); }
  // one batch: the wanted logits, in the order of the entries and of their `want`
  std::vector<float> step(const std::vector<StepEntry>& entries) {
    std::vector<size_t> seqs, counts, want_counts;
    std::vector<uint32_t> tokens, want;
    for (const StepEntry& e : entries) {
      seqs.push_back(e.seq);
      counts.push_back(e.tokens.size());
      want_counts.push_back(e.want.size());
      tokens.insert(tokens.end(), e.tokens.begin(), e.tokens.end());
      want.insert(want.end(), e.want.begin(), e.want.end());
    }
    std::vector<float> logits(want.size() * conf_.vocab_size);
    device_->check(crabml_hip_hybrid_step(ctx_, seqs.size(), seqs.data(), counts.data(), tokens.data(), want_counts.data(), want.data(), logits.data()));
    return logits;
  }
  // greedy steps of several sequences at once: [steps][seqs]
  std::vector<uint32_t> decode_batch(const std::vector<size_t>& seqs, const std::vector<uint32_t>& tokens, size_t steps) {
    if (tokens.size() != seqs.size()) throw Error(ErrorKind::BadInput, "decode_batch: one token per sequence");
    std::vector<uint32_t> out(steps * seqs.size());
    device_->check(crabml_hip_hybrid_decode_greedy(ctx_, seqs.size(), seqs.data(), tokens.data(), steps, out.data()));
    return out;
  }
  // Greedy generation of any number of prompts, steps[i] tokens each.  Up to STEP_ROWS sequences run at a time; prompts that come in
  // together are one batch, sequences decode together in stretches as long as the shortest needs, and a finished one's place (and
  // slab) goes to the next prompt that waits.
  std::vector<std::vector<uint32_t>> generate(const std::vector<std::vector<uint32_t>>& prompts, const std::vector<size_t>& steps) {
    if (steps.size() != prompts.size()) throw Error(ErrorKind::BadInput, "generate: one step count per prompt");
    std::vector<std::vector<uint32_t>> out(prompts.size());
    struct Live {
      size_t request, seq;
    };
    std::vector<Live> live;
    auto give_back = [&]() {
      for (const Live& l : live) (void)crabml_hip_hybrid_close(ctx_, l.seq);
      live.clear();
    };
    try {
      size_t next = 0;
      while (true) {
        std::vector<StepEntry> fresh;
        const size_t first = live.size();
        while (live.size() < STEP_ROWS && next < prompts.size()) {
          if (prompts[next].empty()) throw Error(ErrorKind::BadInput, "generate: expected at least 1 prompt token");
          if (steps[next] == 0) {
            next++;
            continue;
          }
          live.push_back({next, open()});
          fresh.push_back({live.back().seq, prompts[next], {(uint32_t)(prompts[next].size() - 1)}});
          next++;
        }
        if (live.empty()) return out;
        if (!fresh.empty()) {
          const std::vector<float> lg = step(fresh);
          for (size_t i = 0; i < fresh.size(); i++)
            out[live[first + i].request].push_back(
                (uint32_t)sample_argmax(std::vector<float>(lg.begin() + i * conf_.vocab_size, lg.begin() + (i + 1) * conf_.vocab_size)));
        }
        for (size_t i = live.size(); i-- > 0;)
          if (out[live[i].request].size() >= steps[live[i].request]) {
            close(live[i].seq);
            live.erase(live.begin() + (long)i);
          }
        if (live.empty() || (live.size() < STEP_ROWS && next < prompts.size())) continue;
        size_t n = SIZE_MAX;
        std::vector<size_t> seqs;
        std::vector<uint32_t> toks;
        for (const Live& l : live) {
          n = std::min(n, steps[l.request] - out[l.request].size());
          seqs.push_back(l.seq);
          toks.push_back(out[l.request].back());
        }
        const std::vector<uint32_t> ids = decode_batch(seqs, toks, n);
        for (size_t s = 0; s < n; s++)
          for (size_t i = 0; i < live.size(); i++) out[live[i].request].push_back(ids[s * live.size() + i]);
        for (size_t i = live.size(); i-- > 0;)
          if (out[live[i].request].size() >= steps[live[i].request]) {
            close(live[i].seq);
            live.erase(live.begin() + (long)i);
          }
      }
    } catch (...) {
      give_back();
      throw;
    }
  }

  // ---- ModelRunner: one sequence of the runner's own
  const std::string& architecture() const override { return conf_.architecture; }
  size_t vocab_size() const override { return conf_.vocab_size; }
  size_t kv_cache_len() const override { return own_ ? length(*own_) : 0; }
  void reset() override {
    if (own_) close(*own_);
    own_.reset();
  }
  std::vector<float> prefill(const std::vector<uint32_t>& tokens) override {
    if (tokens.empty()) throw Error(ErrorKind::BadInput, "prefill: expected at least 1 prompt token");
    return step({StepEntry{own(), tokens, {(uint32_t)(tokens.size() - 1)}}});
  }
  std::vector<float> forward(size_t token, size_t pos) override {
    if (pos != kv_cache_len()) throw Error(ErrorKind::BadInput, "forward: pos " + std::to_string(pos) + " != sequence length " + std::to_string(kv_cache_len()));
    return step({StepEntry{own(), {(uint32_t)token}, {0}}});
  }
  std::vector<uint32_t> decode_greedy(size_t token, size_t steps) override { return decode_batch({own()}, {(uint32_t)token}, steps); }

 private:
  size_t own() {
    if (!own_) own_ = open();
    return *own_;
  }
  HybridConfig conf_;
  HipTensorDeviceRef device_;
  size_t seq_len_;
  crabml_hip_hybrid_t* ctx_ = nullptr;
  std::optional<size_t> own_;
};

}  // namespace crabml_host
