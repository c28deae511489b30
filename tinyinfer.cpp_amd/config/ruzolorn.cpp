// The Ruzolorn decoder: its config.json read and validated, and the model as data.
//
//   x = embedding.scale * embed[token]; LN(z) = (z - mean) / sqrt(variance + eps) * w, no bias
//   every sublayer has a norm in front and one behind, and what it gives is multiplied by m = residual_mult:
//   x <- x + m LN_1b(mixer(LN_1(x))), x <- x + m LN_2b(ff(LN_2(x)))
//   mixers:  "parallel"   left_scale * left + right_scale * right on the same input.  left (".left.*"): grouped queries, an RMS norm
//                         with a weight on every q and k head (".q.norm", ".k.norm"), no positions, a window of mask.size positions,
//                         softmax of (q . k) scale.  right (".right.*"): Mamba-2, a matrix state per head under a decay that the
//                         token sets, behind a short convolution, a gate in front of a norm in norm_groups parts
//            "retention"  linear attention with a fixed decay per head, the first rot.dims entries of every q and k head rotated, k
//                         times dim^(-1/2), every head's output divided by its root mean square, times silu(W_g h)
//   ff:      "moe": experts W_down (silu(W_gate h) * (W_up h)), softmax scores over experts and identity experts (the last
//            router.identity rows, whose output is h), ".correction" added for the choice only, the largest `top` weighted by their
//            scores as they are, plus a shared expert of the same form; a layer may have none
//   logits = head LN(x) with the weight "final.norm"
//
// Keys: "width", "vocab", "norm": {"eps"}, "embedding": {"scale"}, "residual_mult", "layers": [{"type", "mixer": {...},
// "mlp": {...} | null}].  Tensor names: "embed", "head", "final.norm", "l<i>.norm1 / .norm1b / .norm2 / .norm2b", "l<i>.mix.*",
// "l<i>.mlp.*".
#include "read.h"

namespace tinyinfer {

using namespace config_read;

namespace {
void at_most(int64_t v, int64_t most, const char* key, const std::string& where) {
  if (v > most) throw ConfigError("config.json: " + where + "'" + key + "' (" + std::to_string(v) + ") is not served (up to " + std::to_string(most) + ")");
}
void divides(int64_t part, int64_t whole, const char* part_key, const char* whole_key, const std::string& where) {
  if (whole % part)
    throw ConfigError("config.json: " + where + "'" + whole_key + "' (" + std::to_string(whole) + ") must be a multiple of '" + part_key + "' (" +
                      std::to_string(part) + ")");
}

Json read_left(const Json& m, const std::string& mw) {
  Json o = Json::object();
  const int64_t heads = need_int(m, "heads", mw), dim = need_int(m, "dim", mw);
  const int64_t kv = given(m, "kv_heads") ? need_int(m, "kv_heads", mw) : heads, vdim = given(m, "vdim") ? need_int(m, "vdim", mw) : dim;
  divides(kv, heads, "kv_heads", "heads", mw);
  at_most(dim, 256, "dim", mw);
  at_most(vdim, 256, "vdim", mw);
  o.set("heads", heads);
  o.set("kv_heads", kv);
  o.set("dim", dim);
  o.set("vdim", vdim);
  o.set("scale", given(m, "scale") ? need_float(m, "scale", mw) : 1.0 / std::sqrt((double)dim));
  if (given(m, "mask")) {
    Json mask = Json::object();
    mask.set("size", need_int(m.at("mask"), "size", mw + "mask: "));
    o.set("mask", mask);
  } else {
    o.set("mask", Json());
  }
  return o;
}

Json read_right(const Json& m, const std::string& mw) {
  Json o = Json::object();
  const int64_t heads = need_int(m, "heads", mw), vdim = need_int(m, "vdim", mw), state = need_int(m, "state", mw);
  const int64_t groups = given(m, "groups") ? need_int(m, "groups", mw) : 1, parts = given(m, "norm_groups") ? need_int(m, "norm_groups", mw) : 1;
  divides(groups, heads, "groups", "heads", mw);
  divides(parts, heads * vdim, "norm_groups", "heads * vdim", mw);
  at_most(vdim, 256, "vdim", mw);
  at_most(state, 256, "state", mw);
  o.set("heads", heads);
  o.set("vdim", vdim);
  o.set("state", state);
  o.set("groups", groups);
  o.set("conv", need_int(m, "conv", mw));
  o.set("norm_groups", parts);
  return o;
}

Json read_retention(const Json& m, const std::string& mw) {
  Json o = Json::object();
  const int64_t heads = need_int(m, "heads", mw), dim = need_int(m, "dim", mw), vdim = given(m, "vdim") ? need_int(m, "vdim", mw) : dim;
  at_most(dim, 256, "dim", mw);
  at_most(vdim, 256, "vdim", mw);
  o.set("heads", heads);
  o.set("dim", dim);
  o.set("vdim", vdim);
  if (given(m, "rot")) {
    const std::string rw = mw + "rot: ";
    Json ro = Json::object();
    const int64_t dims = need_int(m.at("rot"), "dims", rw, 0);
    if (dims % 2 || dims > dim)
      throw ConfigError("config.json: " + rw + "'dims' (" + std::to_string(dims) + ") must be even and at most " + std::to_string(dim));
    ro.set("base", need_positive(m.at("rot"), "base", rw));
    ro.set("dims", dims);
    o.set("rot", ro);
  } else {
    o.set("rot", Json());
  }
  const Json& decay = need(m, "decay", mw);
  Json dl = Json::array();
  if (decay.is_number()) {      // one number: every head's
    for (int64_t j = 0; j < heads; ++j) dl.push(Json(decay.as_double()));
  } else {
    if (decay.type() != Json::Array || (int64_t)decay.size() != heads)
      throw ConfigError("config.json: " + mw + "'decay' must list one number a head (" + std::to_string(heads) + ")");
    for (const Json& v : decay.items()) {
      if (!v.is_number()) throw ConfigError("config.json: " + mw + "'decay' must hold numbers, got " + v.dump());
      dl.push(Json(v.as_double()));
    }
  }
  o.set("decay", dl);
  return o;
}

Json read_ff(const Json& e, const std::string& where) {
  Json o = Json::object();
  o.set("ff", need_int(e, "ff", where));
  return o;
}

Json read_moe(const Json& f, const std::string& fw) {
  const std::string kind = given(f, "kind") ? f.at("kind").as_string() : "moe";
  if (kind != "moe") throw ConfigError("config.json: " + fw + "'kind' = '" + kind + "' is not served (moe)");
  Json o = Json::object();
  o.set("kind", kind);
  o.set("expert", read_ff(need(f, "expert", fw), fw + "expert: "));
  const Json& router = need(f, "router", fw);
  const std::string rw = fw + "router: ";
  const int64_t experts = need_int(router, "experts", rw), top = need_int(router, "top", rw);
  const int64_t identity = given(router, "identity") ? need_int(router, "identity", rw, 0) : 0;
  if (top > experts + identity)
    throw ConfigError("config.json: " + rw + "'top' (" + std::to_string(top) + ") exceeds 'experts' and 'identity' (" + std::to_string(experts + identity) + ")");
  Json ro = Json::object();
  ro.set("experts", experts);
  ro.set("top", top);
  ro.set("identity", identity);
  o.set("router", ro);
  o.set("shared", given(f, "shared") ? read_ff(f.at("shared"), fw + "shared: ") : Json());
  return o;
}
}  // namespace

// config.json with every default filled in; ConfigError names the key that is wrong
Json ruzolorn_typed_config(const Json& d) {
  if (d.type() != Json::Object) throw ConfigError("config.json: top level must be a JSON object");
  Json out = Json::object();
  out.set("architecture", "Ruzolorn");
  out.set("width", need_int(d, "width", ""));
  at_most(out.at("width").as_int(), 16384, "width", "");
  out.set("vocab", need_int(d, "vocab", ""));
  Json norm = Json::object();
  norm.set("eps", need_positive(need(d, "norm", ""), "eps", "norm: "));
  out.set("norm", norm);
  Json emb = Json::object();
  emb.set("scale", given(d, "embedding") && given(d.at("embedding"), "scale") ? need_float(d.at("embedding"), "scale", "embedding: ") : 1.0);
  out.set("embedding", emb);
  out.set("residual_mult", given(d, "residual_mult") ? need_float(d, "residual_mult", "") : 1.0);
  const Json& layers = need(d, "layers", "");
  if (layers.type() != Json::Array || layers.size() == 0) throw ConfigError("config.json: 'layers' must be a list of at least one layer");
  Json ls = Json::array();
  for (size_t i = 0; i < layers.size(); ++i) {
    const std::string where = "layers[" + std::to_string(i) + "]: ";
    const Json& l = layers[i];
    if (l.type() != Json::Object) throw ConfigError("config.json: " + where + "must be an object");
    const Json& type = need(l, "type", where);
    const Json& m = need(l, "mixer", where);
    if (type.type() != Json::String || m.type() != Json::Object) throw ConfigError("config.json: " + where + "'type' must be a string and 'mixer' an object");
    Json lo = Json::object(), mo = Json::object();
    lo.set("type", type.as_string());
    const std::string mw = where + "mixer: ";
    if (type.as_string() == "parallel") {
      mo.set("left", read_left(need(m, "left", mw), mw + "left: "));
      mo.set("right", read_right(need(m, "right", mw), mw + "right: "));
      mo.set("left_scale", given(m, "left_scale") ? need_float(m, "left_scale", mw) : 1.0);
      mo.set("right_scale", given(m, "right_scale") ? need_float(m, "right_scale", mw) : 1.0);
    } else if (type.as_string() == "retention") {
      mo = read_retention(m, mw);
    } else {
      throw ConfigError("config.json: " + where + "'type' = '" + type.as_string() + "' is not served (parallel, retention)");
    }
    lo.set("mixer", mo);
    const Json* mlp = l.find("mlp");
    lo.set("mlp", mlp && !mlp->is_null() ? read_moe(*mlp, where + "mlp: ") : Json());
    ls.push(lo);
  }
  out.set("layers", ls);
  return out;
}

ModelSpec ruzolorn_spec(const Json& config) {
  const Json c = ruzolorn_typed_config(config);
  const int64_t H = c.at("width").as_int(), V = c.at("vocab").as_int();
  const double eps = c.at("norm").at("eps").as_double();
  ModelSpec spec;
  spec.architecture = "Ruzolorn";
  spec.vocab_size = V;
  spec.hidden_size = H;
  auto norm = [&](const std::string& tensor) {
    PartSpec p;
    p.kind = "layernorm";
    p.params.set("dim", H);
    p.params.set("eps", eps);
    p.params.set("tensor", tensor);
    return p;
  };
  auto left_mixer = [&](const Json& m, const std::string& at) {
    PartSpec p;
    p.kind = "attention";
    p.name = "left";
    p.params.set("hidden", H);
    p.params.set("heads", m.at("heads").as_int());
    p.params.set("kv_heads", m.at("kv_heads").as_int());
    p.params.set("head_dim", m.at("dim").as_int());
    p.params.set("v_head_dim", m.at("vdim").as_int());
    p.params.set("scale", m.at("scale").as_double());
    p.params.set("eps", eps);
    p.params.set("general", true);      // it writes apart from the residual whatever its sizes
    p.params.set("qk_norm", true);
    p.params.set("q_norm", at + ".q.norm");
    p.params.set("k_norm", at + ".k.norm");
    if (m.has("mask")) p.params.set("window", m.at("mask").at("size").as_int());
    for (const char* t : {"q", "k", "v", "o"}) p.params.set(t, at + "." + t);
    return p;
  };
  auto right_mixer = [&](const Json& m) {
    PartSpec p;
    p.kind = "mamba2";
    p.name = "right";
    p.params.set("hidden", H);
    p.params.set("eps", eps);
    p.params.set("v_head_dim", m.at("vdim").as_int());
    for (const char* key : {"heads", "state", "groups", "conv", "norm_groups"}) p.params.set(key, m.at(key).as_int());
    return p;
  };
  spec.embedding.kind = "table";
  spec.embedding.params.set("vocab", V);
  spec.embedding.params.set("dim", H);
  spec.embedding.params.set("tensor", "embed");
  spec.embedding.params.set("scale", c.at("embedding").at("scale").as_double());
  const Json& layers = c.at("layers");
  for (size_t i = 0; i < layers.size(); ++i) {
    const Json& l = layers[i];
    const Json& m = l.at("mixer");
    LayerSpec ls;
    ls.prefix = "l" + std::to_string(i);
    ls.block.kind = "sandwich";
    ls.block.params.set("factor", c.at("residual_mult").as_double());
    ls.block.params.set("defer_write", i + 1 < layers.size());      // the next layer's first read takes the last write in
    ls.parts.emplace_back("norm1", norm(ls.prefix + ".norm1"));
    PartSpec mix;
    mix.params.set("hidden", H);
    if (l.at("type").as_string() == "parallel") {
      mix.kind = "sum";
      mix.params.set("left", left_mixer(m.at("left"), ls.prefix + ".mix.left").to_json());
      mix.params.set("right", right_mixer(m.at("right")).to_json());
      mix.params.set("left_scale", m.at("left_scale").as_double());
      mix.params.set("right_scale", m.at("right_scale").as_double());
    } else {
      mix.kind = "decay_attention";
      mix.params.set("heads", m.at("heads").as_int());
      mix.params.set("head_dim", m.at("dim").as_int());
      mix.params.set("v_head_dim", m.at("vdim").as_int());
      mix.params.set("decay", m.at("decay"));
      mix.params.set("eps", eps);
      mix.params.set("activation", "none");
      mix.params.set("k_scale", 1.0 / std::sqrt((double)m.at("dim").as_int()));
      mix.params.set("norm", "head");
      mix.params.set("gate", "silu");
      if (m.has("rot") && m.at("rot").at("dims").as_int() > 0) {
        PartSpec pos;
        pos.kind = "rope_partial";
        pos.params = m.at("rot");
        mix.params.set("pos", pos.to_json());
      }
    }
    mix.name = "mix";
    ls.parts.emplace_back("mixer", mix);
    ls.parts.emplace_back("norm1b", norm(ls.prefix + ".norm1b"));
    if (l.has("mlp")) {
      const Json& f = l.at("mlp");
      const Json& r = f.at("router");
      ls.parts.emplace_back("norm2", norm(ls.prefix + ".norm2"));
      PartSpec ff;
      ff.kind = "moe";
      ff.name = "mlp";
      ff.params.set("hidden", H);
      ff.params.set("intermediate", f.at("expert").at("ff").as_int());
      for (const char* key : {"experts", "top", "identity"}) ff.params.set(key, r.at(key).as_int());
      ff.params.set("activation", "glu_silu");
      ff.params.set("score", "softmax");
      ff.params.set("renormalize", false);
      ff.params.set("correction", true);
      if (f.has("shared")) {
        PartSpec sh;
        sh.kind = "glu";
        sh.name = "shared";
        sh.params.set("hidden", H);
        sh.params.set("intermediate", f.at("shared").at("ff").as_int());
        ff.params.set("shared", sh.to_json());
      }
      ls.parts.emplace_back("ffn", ff);
      ls.parts.emplace_back("norm2b", norm(ls.prefix + ".norm2b"));
    } else {      // the norms around a feed-forward that is not there may lie in the checkpoint all the same
      Json spare = Json::array();
      for (const char* t : {".norm2", ".norm2b"}) spare.push(Json(ls.prefix + t));
      ls.block.params.set("spare", spare);
      ls.block.params.set("dim", H);
    }
    spec.layers.push_back(std::move(ls));
  }
  spec.final_norm = norm("final.norm");
  spec.lm_head.kind = "linear";
  spec.lm_head.params.set("vocab", V);
  spec.lm_head.params.set("dim", H);
  spec.lm_head.params.set("tied", false);
  spec.lm_head.params.set("tensor", "head");
  return spec;
}

}  // namespace tinyinfer
