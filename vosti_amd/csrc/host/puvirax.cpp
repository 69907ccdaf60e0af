#include "puvirax.h"

#include "config_read.h"

namespace vosti {
namespace {

constexpr int64_t kMaxPositions = 1 << 22;  // the angles are computed, not tabulated; this bounds a request's length

// A rotation by computed angles of entries i and i + dims / 2 of a head's first `dims`, with frequencies by bands of their
// wavelength where there is a 'scaling'.
PartSpecPtr rotation(const Json& rot, int64_t dim, const std::string& where) {
  const int64_t dims = config_positive(rot, "dims", where + " rot");
  const double base = config_number(rot, "base", where + " rot");
  if (dims % 2 || dims > dim) throw ConfigError("config.json: " + where + ": 'rot.dims' must be even and at most 'dim'");
  if (base <= 0.0) throw ConfigError("config.json: " + where + ": 'rot.base' must be positive");
  std::map<std::string, double> n = {{"head_dim", (double)dim}, {"rotary_dim", (double)dims}, {"theta", base}, {"max_positions", (double)kMaxPositions}};
  if (const Json* s = rot.get("scaling")) {
    const std::pair<const char*, const char*> keys[] = {{"band_factor", "factor"}, {"original", "original"}, {"band_low", "low"}, {"band_high", "high"}};
    for (const auto& k : keys) {
      n[k.first] = config_number(*s, k.second, where + " rot.scaling");
      if (n[k.first] <= 0) throw ConfigError("config.json: " + where + ": 'rot.scaling." + k.second + "' must be positive");
    }
    if (n["band_low"] > n["band_high"]) throw ConfigError("config.json: " + where + ": 'rot.scaling.low' must not exceed 'rot.scaling.high'");
  }
  return make_part("rotary_stretched", n);
}

// mixes: 0 (the values stay as they are), 1 (the first layer that mixes: its values are kept), 2 (they are blended with those).
PartSpecPtr attention_mixer(const std::string& type, const Json& m, int mixes, int64_t width, double eps, const std::string& where, const std::string& p,
                            LayerSpec& ls) {
  const int64_t heads = config_positive(m, "heads", where), kv_heads = config_positive(m, "kv_heads", where);
  const int64_t dim = config_positive(m, "dim", where), vdim = config_positive(m, "vdim", where);
  if (heads % kv_heads) throw ConfigError("config.json: " + where + ": 'heads' must be a multiple of 'kv_heads'");
  const double scale = config_number(m, "scale", where);
  if (scale <= 0) throw ConfigError("config.json: " + where + ": 'scale' must be positive");
  std::map<std::string, double> n = {{"hidden_size", (double)width}, {"num_heads", (double)heads}, {"num_kv_heads", (double)kv_heads},
                                     {"head_dim", (double)dim}, {"value_dim", (double)vdim}, {"scale", scale}, {"exact_weights", 1.0},
                                     {"value_mix", (double)mixes}};
  std::map<std::string, PartSpecPtr> below;
  for (const char* t : {"q", "k", "v", "o"}) ls.names[std::string("mixer.") + t + "_proj.weight"] = p + "mix." + t;
  if (mixes == 2) ls.names["mixer.value_share"] = p + "mix.vmix";
  if (type == "attention") {
    n["unit_norm"] = 1.0;
    n["eps"] = eps;
    n["head_gate"] = 1.0;
    below["position"] = rotation(config_member(m, "rot", where), dim, where);
    ls.names["mixer.head_gate.weight"] = p + "mix.g";
  } else {
    const bool whole = type == "attention_3";
    if (whole) n["whole_norm"] = 1.0;
    else if (const Json* mask = m.get("mask")) n["window"] = (double)config_positive(*mask, "size", where + " mask");
    below["q_norm"] = make_part("rmsnorm", {{"size", (double)(whole ? heads * dim : dim)}, {"eps", eps}});
    below["k_norm"] = make_part("rmsnorm", {{"size", (double)(whole ? kv_heads * dim : dim)}, {"eps", eps}});
    n["distance_bias"] = 1.0;
    n["bias_max"] = config_number(m, "bias_max", where);
    if (n["bias_max"] <= 0) throw ConfigError("config.json: " + where + ": 'bias_max' must be positive");
    for (const char* t : {"q", "k"}) ls.names[std::string("mixer.") + t + "_norm.weight"] = p + "mix." + t + ".norm";
    ls.names["mixer.distance_bias"] = p + "mix.rel";
  }
  return make_part("attention", n, below);
}

PartSpecPtr feed_forward(const Json& mlp, int64_t width, const std::string& where, const std::string& p, LayerSpec& ls) {
  const std::string kind = config_text(mlp, "kind", where);
  if (kind == "dense") {
    for (const char* w : {"up", "down"}) ls.names[std::string("feed_forward.") + w + "_proj.weight"] = p + "mlp." + w;
    return make_part("squared_relu", {{"hidden_size", (double)width}, {"intermediate_size", (double)config_positive(mlp, "ff", where)}});
  }
  if (kind != "moe") throw ConfigError("config.json: " + where + ": 'kind' must be 'dense' or 'moe'");
  const Json& router = config_member(mlp, "router", where);
  const std::string rw = where + ".router";
  const int64_t experts = config_positive(router, "experts", rw), top = config_positive(router, "top", rw);
  int64_t groups = 1, keep = 1;
  if (const Json* g = router.get("groups")) {
    groups = config_positive(*g, "count", rw + ".groups");
    keep = config_positive(*g, "keep", rw + ".groups");
  }
  if (experts % groups) throw ConfigError("config.json: " + rw + ": 'groups.count' must divide 'experts'");
  if (keep > groups) throw ConfigError("config.json: " + rw + ": 'groups.keep' must not exceed 'groups.count'");
  if (top > keep * (experts / groups)) throw ConfigError("config.json: " + rw + ": 'top' must not exceed the experts of the kept groups");
  const int64_t ff = config_positive(config_member(mlp, "expert", where), "ff", where + ".expert");
  // score 1: logistic scores, not divided by anything; the correction joins them for the choice alone; a group is worth the sum
  // of its two largest.
  std::map<std::string, double> n = {{"hidden_size", (double)width}, {"intermediate_size", (double)ff}, {"experts", (double)experts}, {"top", (double)top},
                                     {"score", 1.0}, {"choice_correction", 1.0}, {"groups", (double)groups}, {"keep_groups", (double)keep},
                                     {"group_score", 1.0}};
  ls.names["feed_forward.router.weight"] = p + "mlp.router";
  ls.names["feed_forward.router.correction"] = p + "mlp.correction";
  for (int64_t e = 0; e < experts; ++e) {
    const std::string en = std::to_string(e);
    for (const char* w : {"up", "down"}) ls.names["feed_forward.experts." + en + "." + w + "_proj.weight"] = p + "mlp.e" + en + "." + w;
  }
  if (const Json* shared = mlp.get("shared")) {
    n["shared_size"] = (double)config_positive(*shared, "ff", where + ".shared");
    for (const char* w : {"up", "down"}) ls.names[std::string("feed_forward.shared.") + w + "_proj.weight"] = p + "mlp.shared." + w;
  }
  return make_part("routed_experts", n);
}

}  // namespace

ModelSpec puvirax_model_spec(const Json& raw) {
  const int64_t width = config_positive(raw, "width", "the model's"), vocab = config_positive(raw, "vocab", "the model's");
  const double eps = config_number(config_member(raw, "norm", "the model"), "eps", "norm");
  if (eps < 0) throw ConfigError("config.json: 'norm.eps' must not be negative");
  const double logit_scale = raw.get("logit_scale") ? config_number(raw, "logit_scale", "the model's") : 1.0;
  const Json& layers = config_member(raw, "layers", "the model");
  if (layers.kind != Json::Array) throw ConfigError("config.json: 'layers' must be a list");
  const int64_t L = (int64_t)layers.items.size();
  const PartSpecPtr norm = make_part("rmsnorm", {{"size", (double)width}, {"eps", eps}});

  ModelSpec spec;
  spec.architecture = "Puvirax";
  spec.vocab_size = vocab;
  spec.hidden_size = width;
  spec.max_positions = kMaxPositions;
  spec.names = {{"embedding.weight", "embed"}, {"final_norm.weight", "final.norm"}, {"head.weight", "embed"}};
  const Json* embedding = raw.get("embedding");
  int64_t buckets = 0;
  if (const Json* b = embedding ? embedding->get("bigram") : nullptr) {
    buckets = config_positive(*b, "buckets", "embedding.bigram");
    std::map<std::string, double> n = {{"vocab_size", (double)vocab}, {"hidden_size", (double)width}, {"buckets", (double)buckets}};
    for (const char* key : {"mul_prev", "mul_cur"}) {
      const Json& v = config_member(*b, key, "embedding.bigram");
      if (!v.is_int() || v.as_int() < 0 || v.as_int() >= (1ll << 31)) throw ConfigError(std::string("config.json: embedding.bigram '") + key + "' must be an integer from 0 below 2^31");
      n[key] = (double)v.as_int();
    }
    spec.embedding = make_part("token_embedding_bigram", n);
    spec.names["embedding.bigram"] = "bigram";
  } else {
    spec.embedding = make_part("token_embedding_scaled", {{"vocab_size", (double)vocab}, {"hidden_size", (double)width}, {"scale", 1.0}});
  }
  // The constant on the logits goes into the norm before the projection: one multiplication of its 32-bit weight.
  spec.final_norm = make_part("rmsnorm", {{"size", (double)width}, {"eps", eps}, {"scale", logit_scale}});
  spec.head = make_part("linear_head", {{"vocab_size", (double)vocab}, {"hidden_size", (double)width}});

  int64_t first_mixing = -1, mixed_entries = 0;
  for (int64_t i = 0; i < L; ++i) {
    const Json& l = layers.items[i];
    const std::string where = "layer " + std::to_string(i), p = "l" + std::to_string(i) + ".", type = config_text(l, "type", where);
    if (type != "attention" && type != "attention_2" && type != "attention_3") throw ConfigError("config.json: " + where + ": unknown mixer type '" + type + "'");
    const Json& m = config_member(l, "mixer", where);
    int mixes = 0;
    if (const Json* mix = m.get("v_mix")) {
      if (mix->kind != Json::Bool) throw ConfigError("config.json: " + where + ": 'v_mix' must be true or false");
      if (mix->boolean) mixes = first_mixing < 0 ? 1 : 2;
    }
    if (mixes) {
      const int64_t entries = config_positive(m, "kv_heads", where) * config_positive(m, "vdim", where);
      if (mixes == 1) {
        first_mixing = i;
        mixed_entries = entries;
      } else if (entries != mixed_entries) {
        throw ConfigError("config.json: " + where + ": its " + std::to_string(entries) + " values a token cannot be blended with the " +
                          std::to_string(mixed_entries) + " of layer " + std::to_string(first_mixing));
      }
    }
    // A layer that blends nothing may hold its share all the same.
    if (mixes != 2) spec.ignored_names.push_back(p + "mix.vmix");
    LayerSpec ls;
    ls.block = "prenorm";
    ls.norms = {{"input", norm}};
    ls.names = {{"norms.input.weight", p + "norm1"}};
    ls.mixer = attention_mixer(type, m, mixes, width, eps, where, p, ls);
    if (const Json* mlp = l.get("mlp")) {
      ls.feed_forward = feed_forward(*mlp, width, where + " mlp", p, ls);
      ls.norms["post_mixer"] = norm;
      ls.names["norms.post_mixer.weight"] = p + "norm2";
    } else {
      ls.feed_forward = make_part("none", {});
      spec.ignored_names.push_back(p + "norm2");      // nothing to stand before; a checkpoint may still hold the weight
    }
    spec.layers.push_back(std::move(ls));
    spec.schedule.push_back({(int)i, -1});
  }
  spec.config_json = "{\"vocab\": " + std::to_string(vocab) + ", \"width\": " + std::to_string(width) + ", \"layers\": " + std::to_string(L) +
                     ", \"norm_eps\": " + json_number(eps) + ", \"logit_scale\": " + json_number(logit_scale) + ", \"bigram_buckets\": " +
                     std::to_string(buckets) + "}";
  return spec;
}

}  // namespace vosti
