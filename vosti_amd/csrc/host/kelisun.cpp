#include "kelisun.h"

#include "config_read.h"

namespace vosti {
namespace {

constexpr int64_t kMaxPositions = 1 << 22;  // the angles are computed, not tabulated; this bounds a request's length

// A rotation by computed angles of entries i and i + dims / 2, whose long wavelengths 'scaling' stretches (absent: none).
PartSpecPtr rotation(const Json& rot, int64_t size, const std::string& where) {
  const int64_t dims = config_positive(rot, "dims", where + " rot");
  const double base = config_number(rot, "base", where + " rot");
  if (dims != size || dims % 2) throw ConfigError("config.json: " + where + ": 'rot.dims' must be even and equal 'rot_dim'");
  if (base <= 1.0) throw ConfigError("config.json: " + where + ": 'rot.base' must be larger than 1");
  std::map<std::string, double> n = {{"head_dim", (double)size}, {"rotary_dim", (double)dims}, {"theta", base}, {"max_positions", (double)kMaxPositions}};
  if (const Json* s = rot.get("scaling")) {
    for (const char* key : {"factor", "original", "fast", "slow"}) {
      n[key] = config_number(*s, key, where + " rot.scaling");
      if (n[key] <= 0) throw ConfigError("config.json: " + where + ": 'rot.scaling." + key + "' must be positive");
    }
  }
  return make_part("rotary_stretched", n);
}

PartSpecPtr latent_mixer(const Json& m, int64_t width, double eps, const std::string& where, const std::string& p, LayerSpec& ls) {
  const int64_t heads = config_positive(m, "heads", where), dim = config_positive(m, "dim", where), rot_dim = config_positive(m, "rot_dim", where);
  const int64_t vdim = config_positive(m, "vdim", where), kv_rank = config_positive(m, "kv_rank", where);
  const double scale = config_number(m, "scale", where);
  if (scale <= 0) throw ConfigError("config.json: " + where + ": 'scale' must be positive");
  const int64_t window = m.get("mask") ? config_positive(*m.get("mask"), "size", where + " mask") : 0;
  const std::pair<const char*, const char*> names[] = {{"q_proj.weight", "q"}, {"kv_down.weight", "dkv"}, {"kv_down_norm.weight", "dkv.norm"},
                                                       {"k_up.weight", "uk"},  {"v_up.weight", "uv"},     {"sinks", "sink"},
                                                       {"o_proj.weight", "o"}};
  for (const auto& n : names) ls.names[std::string("mixer.") + n.first] = p + "mix." + n.second;
  return make_part("latent_attention", {{"hidden_size", (double)width}, {"num_heads", (double)heads}, {"head_dim", (double)dim},
                                        {"rotary_dim", (double)rot_dim}, {"value_dim", (double)vdim}, {"kv_rank", (double)kv_rank}, {"q_rank", 0.0},
                                        {"scale", scale}, {"eps", eps}, {"own_kv", 1.0}, {"window", (double)window}, {"sink", 1.0}},
                   {{"position", rotation(config_member(m, "rot", where), rot_dim, where)}});
}

PartSpecPtr expert_mixture(const Json& mlp, int64_t width, const std::string& where, const std::string& p, LayerSpec& ls) {
  if (config_text(mlp, "kind", where) != "moe") throw ConfigError("config.json: " + where + ": 'kind' must be 'moe'");
  const Json& router = config_member(mlp, "router", where);
  const std::string rw = where + ".router";
  const int64_t experts = config_positive(router, "experts", rw), top = config_positive(router, "top", rw);
  const double scale = router.get("scale") ? config_number(router, "scale", rw) : 1.0;
  int64_t groups = 1, keep = 1;
  if (const Json* g = router.get("groups")) {
    groups = config_positive(*g, "count", rw + ".groups");
    keep = config_positive(*g, "keep", rw + ".groups");
  }
  if (experts % groups) throw ConfigError("config.json: " + rw + ": 'groups.count' must divide 'experts'");
  if (keep > groups) throw ConfigError("config.json: " + rw + ": 'groups.keep' must not exceed 'groups.count'");
  if (top > keep * (experts / groups)) throw ConfigError("config.json: " + rw + ": 'top' must not exceed the experts of the kept groups");
  const int64_t ff = config_positive(config_member(mlp, "expert", where), "ff", where + ".expert");
  ls.names["feed_forward.router.weight"] = p + "mlp.router";
  for (int64_t e = 0; e < experts; ++e) {
    const std::string en = std::to_string(e);
    for (const char* w : {"gate", "up", "down"}) ls.names["feed_forward.experts." + en + "." + w + "_proj.weight"] = p + "mlp.e" + en + "." + w;
  }
  // gated without a limit, slope 1 and shift 0: silu(gate) * up.  score 2: the softmax scores as they are.
  return make_part("routed_experts", {{"hidden_size", (double)width}, {"intermediate_size", (double)ff}, {"experts", (double)experts}, {"top", (double)top},
                                      {"gated", 1.0}, {"score", 2.0}, {"groups", (double)groups}, {"keep_groups", (double)keep}, {"weight_scale", scale}});
}

}  // namespace

ModelSpec kelisun_model_spec(const Json& raw) {
  const int64_t width = config_positive(raw, "width", "the model's"), vocab = config_positive(raw, "vocab", "the model's");
  const int64_t streams = config_positive(raw, "streams", "the model's");
  const double eps = config_number(config_member(raw, "norm", "the model"), "eps", "norm");
  if (eps < 0) throw ConfigError("config.json: 'norm.eps' must not be negative");
  const Json& layers = config_member(raw, "layers", "the model");
  if (layers.kind != Json::Array) throw ConfigError("config.json: 'layers' must be a list");
  const int64_t L = (int64_t)layers.items.size();
  const PartSpecPtr norm = make_part("rmsnorm", {{"size", (double)width}, {"eps", eps}});

  ModelSpec spec;
  spec.architecture = "Kelisun";
  spec.vocab_size = vocab;
  spec.hidden_size = width;
  spec.max_positions = kMaxPositions;
  spec.embedding = make_part("token_embedding_normed", {{"vocab_size", (double)vocab}, {"hidden_size", (double)width}, {"eps", eps}});
  spec.final_norm = norm;
  spec.head = make_part("linear_head", {{"vocab_size", (double)vocab}, {"hidden_size", (double)width}});
  spec.names = {{"embedding.weight", "embed"}, {"embedding.norm.weight", "embed.norm"}, {"final_norm.weight", "final.norm"}, {"head.weight", "head"}};

  // The layers that have tensors of their own, in order; the others run one of these a second time.
  std::map<int64_t, int> built;          // entry -> its place in spec.layers
  for (int64_t i = 0; i < L; ++i) {
    const Json& l = layers.items[i];
    if (l.get("weights_of")) continue;
    const std::string where = "layer " + std::to_string(i), p = "l" + std::to_string(i) + ".";
    if (config_text(l, "type", where) != "latent_attention") throw ConfigError("config.json: " + where + ": unknown mixer type '" + l.get("type")->text + "'");
    LayerSpec ls;
    ls.block = "hyper_streams";
    ls.block_numbers = {{"hidden_size", (double)width}, {"streams", (double)streams}};
    ls.norms = {{"mixer_in", norm}};
    ls.names = {{"norms.mixer_in.weight", p + "norm1"}};
    for (const char* c : {"in", "out", "mix"}) ls.names[std::string("hyper_mixer.") + c] = p + "hc1." + c;
    ls.mixer = latent_mixer(config_member(l, "mixer", where), width, eps, where, p, ls);
    if (const Json* mlp = l.get("mlp")) {
      ls.feed_forward = expert_mixture(*mlp, width, where + " mlp", p, ls);
      ls.norms["ffn_in"] = norm;
      ls.names["norms.ffn_in.weight"] = p + "norm2";
      for (const char* c : {"in", "out", "mix"}) ls.names[std::string("hyper_ffn.") + c] = p + "hc2." + c;
    } else {
      // Nothing follows the mixer; a checkpoint may still hold the second sublayer's norm and coefficients.
      ls.feed_forward = make_part("none", {});
      for (const char* n : {"norm2", "hc2.in", "hc2.out", "hc2.mix"}) spec.ignored_names.push_back(p + n);
    }
    built[i] = (int)spec.layers.size();
    spec.layers.push_back(std::move(ls));
  }
  for (int64_t i = 0; i < L; ++i) {
    int64_t from = i;
    for (int64_t hops = 0; const Json* of = layers.items[from].get("weights_of"); ++hops) {
      const std::string where = "layer " + std::to_string(from);
      if (!of->is_int() || of->as_int() < 0 || of->as_int() >= L || hops >= L)
        throw ConfigError("config.json: " + where + ": 'weights_of' must lead to a layer with weights of its own");
      if (!same_config(layers.items[from], layers.items[of->as_int()], "weights_of"))
        throw ConfigError("config.json: " + where + " differs from the layer whose weights it uses");
      from = of->as_int();
    }
    spec.schedule.push_back({built.at(from), -1});
  }
  spec.config_json = "{\"vocab\": " + std::to_string(vocab) + ", \"width\": " + std::to_string(width) + ", \"layers\": " + std::to_string(L) +
                     ", \"streams\": " + std::to_string(streams) + ", \"norm_eps\": " + json_number(eps) + "}";
  return spec;
}

}  // namespace vosti
