// What the readers of config.json share: keys that must be there, with a type and a range, refused by name.
#pragma once
#include <cmath>
#include <string>

#include "../include/inference.h"

namespace tinyinfer {
namespace config_read {
inline const Json& need(const Json& d, const char* key, const std::string& where) {
  const Json* v = d.type() == Json::Object ? d.find(key) : nullptr;
  if (!v || v->is_null()) throw ConfigError("config.json: " + where + "'" + key + "' is missing");
  return *v;
}
inline int64_t need_int(const Json& d, const char* key, const std::string& where, int64_t least = 1) {
  const Json& v = need(d, key, where);
  const bool whole = v.type() == Json::Int || (v.type() == Json::Float && v.as_double() == std::floor(v.as_double()));
  if (!whole) throw ConfigError("config.json: " + where + "'" + key + "' must be an integer, got " + v.dump());
  if (v.as_int() < least)
    throw ConfigError("config.json: " + where + "'" + key + "' must be at least " + std::to_string(least) + ", got " + v.dump());
  return v.as_int();
}
inline double need_float(const Json& d, const char* key, const std::string& where) {
  const Json& v = need(d, key, where);
  if (!v.is_number()) throw ConfigError("config.json: " + where + "'" + key + "' must be a number, got " + v.dump());
  return v.as_double();
}
inline double need_positive(const Json& d, const char* key, const std::string& where) {
  const double v = need_float(d, key, where);
  if (!(v > 0.0)) throw ConfigError("config.json: " + where + "'" + key + "' must be positive");
  return v;
}
inline bool given(const Json& d, const char* key) { return d.type() == Json::Object && d.has(key); }
}  // namespace config_read
}  // namespace tinyinfer
