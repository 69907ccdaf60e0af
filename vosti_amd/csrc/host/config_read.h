// Reading a configuration's members, with errors that name the key and where it is missing or wrong.
#pragma once
#include <cmath>
#include <cstdint>
#include <map>
#include <memory>
#include <string>

#include "spec.h"

namespace vosti {

inline PartSpecPtr make_part(std::string kind, std::map<std::string, double> numbers, std::map<std::string, PartSpecPtr> parts = {}) {
  auto p = std::make_shared<PartSpec>();
  p->kind = std::move(kind);
  p->numbers = std::move(numbers);
  for (auto& c : parts) p->parts[c.first] = c.second;
  return p;
}

inline const Json& config_member(const Json& j, const std::string& key, const std::string& where) {
  const Json* v = j.get(key);
  if (!v) throw ConfigError("config.json: " + where + " lacks '" + key + "'");
  return *v;
}

inline int64_t config_positive(const Json& j, const std::string& key, const std::string& where) {
  const Json& v = config_member(j, key, where);
  if (!v.is_int() || v.as_int() <= 0) throw ConfigError("config.json: " + where + " '" + key + "' must be a positive integer");
  return v.as_int();
}

inline double config_number(const Json& j, const std::string& key, const std::string& where) {
  const Json& v = config_member(j, key, where);
  if (v.kind != Json::Number || !std::isfinite(v.number)) throw ConfigError("config.json: " + where + " '" + key + "' must be a finite number");
  return v.number;
}

inline std::string config_text(const Json& j, const std::string& key, const std::string& where) {
  const Json& v = config_member(j, key, where);
  if (v.kind != Json::String) throw ConfigError("config.json: " + where + " '" + key + "' must be a string");
  return v.text;
}

// Whether two values mean the same: numbers by value, objects whatever the order of their members; a member that is null is
// as good as absent, and so is one of the first object's that `except` names.
inline bool same_config(const Json& a, const Json& b, const std::string& except = "") {
  if (a.kind != b.kind) return false;
  switch (a.kind) {
    case Json::Null: return true;
    case Json::Bool: return a.boolean == b.boolean;
    case Json::Number: return a.number == b.number;
    case Json::String: return a.text == b.text;
    case Json::Array:
      if (a.items.size() != b.items.size()) return false;
      for (size_t i = 0; i < a.items.size(); ++i)
        if (!same_config(a.items[i], b.items[i])) return false;
      return true;
    case Json::Object:
      for (const auto& m : a.members)
        if (m.first != except && !m.second.is_null() && !(b.get(m.first) && same_config(m.second, *b.get(m.first)))) return false;
      for (const auto& m : b.members)
        if (m.first != except && !m.second.is_null() && !a.get(m.first)) return false;
      return true;
  }
  return false;
}

}  // namespace vosti
