// The Lupolorn decoder: its config.json read and validated, and the model as data.
//
//   x = embedding.scale * embed[token]; rms(z) = sqrt(mean(z^2) + eps), a norm: z / rms(z) * w
//   every sublayer has a norm in front and one behind: x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(norm2(x)))
//   mixers:  "mingru"            s = sigmoid(W_z h + b_z), u = W_x h + b_x, c = u + 1/2 (u >= 0) or sigmoid(u);
//                                S_t = (1 - s) S_(t-1) + s c element by element; W_o (S_t * silu(W_g h))
//            "latent_attention"  queries W_uq norm(W_dq h), keys W_uk c and values W_uv c per head from the cached latent
//                                c = norm(W_dkv h); no positions; a window of mask.size positions; softmax of (q . k) scale
//            "attention"         grouped queries; the first rot.dims entries of a head rotated, neighbours in pairs, the
//                                frequencies stretched by wavelength (rot.scaling); then q and k divided by their rms; causal
//                                softmax of (q . k) scale with one more in its denominator; a sigmoid gate a head (".g")
//   ff:      "dense"  W_down relu(W_up h)^2;  "moe": experts of that form, softmax scores, the largest `top` chosen, weighted by
//            their scores as they are, plus a shared expert times sigmoid(W_sg h); a layer may have none
//   logits = embed norm(x) with the weight "final.norm"
//
// Keys: "width", "vocab", "norm": {"eps"}, "embedding": {"scale"}, "layers": [{"type", "mixer": {...}, "mlp": {...} | null}].
// Tensor names: "embed", "final.norm", "l<i>.norm1 / .norm1b / .norm2 / .norm2b", "l<i>.mix.*", "l<i>.mlp.*".
#include "read.h"

namespace tinyinfer {

using namespace config_read;

namespace {
// "rot": {"base", "dims", "scaling": {factor, low, high, original} | absent} or absent; `most`: the entries a head has to turn
Json read_rot(const Json& m, const std::string& mw, int64_t most) {
  if (!given(m, "rot")) return Json();
  const Json& r = m.at("rot");
  const std::string rw = mw + "rot: ";
  Json ro = Json::object();
  const int64_t dims = need_int(r, "dims", rw, 0);
  if (dims % 2 || dims > most)
    throw ConfigError("config.json: " + rw + "'dims' (" + std::to_string(dims) + ") must be even and at most " + std::to_string(most));
  ro.set("base", need_positive(r, "base", rw));
  ro.set("dims", dims);
  if (given(r, "scaling")) {
    Json so = Json::object();
    for (const char* key : {"factor", "low", "high", "original"}) so.set(key, need_positive(r.at("scaling"), key, rw + "scaling: "));
    if (so.at("low").as_double() > so.at("high").as_double())
      throw ConfigError("config.json: " + rw + "scaling: 'low' must not exceed 'high'");
    ro.set("scaling", so);
  } else {
    ro.set("scaling", Json());
  }
  return ro;
}

Json read_ff(const Json& e, const std::string& where) {
  Json o = Json::object();
  o.set("ff", need_int(e, "ff", where));
  return o;
}
}  // namespace

// config.json with every default filled in; ConfigError names the key that is wrong
Json lupolorn_typed_config(const Json& d) {
  if (d.type() != Json::Object) throw ConfigError("config.json: top level must be a JSON object");
  Json out = Json::object();
  out.set("architecture", "Lupolorn");
  out.set("width", need_int(d, "width", ""));
  out.set("vocab", need_int(d, "vocab", ""));
  Json norm = Json::object();
  norm.set("eps", need_positive(need(d, "norm", ""), "eps", "norm: "));
  out.set("norm", norm);
  Json emb = Json::object();
  emb.set("scale", given(d, "embedding") && given(d.at("embedding"), "scale") ? need_float(d.at("embedding"), "scale", "embedding: ") : 1.0);
  out.set("embedding", emb);
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
    if (type.as_string() == "mingru") {
      mo.set("width", need_int(m, "width", mw));
    } else if (type.as_string() == "attention" || type.as_string() == "latent_attention") {
      const bool latent = type.as_string() == "latent_attention";
      const int64_t heads = need_int(m, "heads", mw), dim = need_int(m, "dim", mw);
      mo.set("heads", heads);
      mo.set("dim", dim);
      mo.set("vdim", given(m, "vdim") ? need_int(m, "vdim", mw) : dim);
      mo.set("scale", given(m, "scale") ? need_float(m, "scale", mw) : 1.0 / std::sqrt((double)dim));
      if (latent) {
        mo.set("q_rank", need_int(m, "q_rank", mw));
        mo.set("kv_rank", need_int(m, "kv_rank", mw));
        if (given(m, "mask")) {
          Json mask = Json::object();
          mask.set("size", need_int(m.at("mask"), "size", mw + "mask: "));
          mo.set("mask", mask);
        } else {
          mo.set("mask", Json());
        }
      } else {
        const int64_t kv = given(m, "kv_heads") ? need_int(m, "kv_heads", mw) : heads;
        if (heads % kv) throw ConfigError("config.json: " + mw + "'heads' (" + std::to_string(heads) + ") must be a multiple of 'kv_heads' (" + std::to_string(kv) + ")");
        if (dim > 256) throw ConfigError("config.json: " + mw + "'dim' (" + std::to_string(dim) + ") is not served (up to 256)");
        if (mo.at("vdim").as_int() > 256) throw ConfigError("config.json: " + mw + "'vdim' is not served (up to 256)");
        mo.set("kv_heads", kv);
        mo.set("rot", read_rot(m, mw, dim));
      }
    } else {
      throw ConfigError("config.json: " + where + "'type' = '" + type.as_string() + "' is not served (attention, latent_attention, mingru)");
    }
    lo.set("mixer", mo);
    const Json* mlp = l.find("mlp");
    if (mlp && !mlp->is_null()) {
      const std::string fw = where + "mlp: ";
      const std::string kind = given(*mlp, "kind") ? need(*mlp, "kind", fw).as_string() : "dense";
      Json fo = Json::object();
      fo.set("kind", kind);
      if (kind == "dense") {
        fo.set("ff", need_int(*mlp, "ff", fw));
      } else if (kind == "moe") {
        fo.set("expert", read_ff(need(*mlp, "expert", fw), fw + "expert: "));
        const Json& router = need(*mlp, "router", fw);
        const int64_t experts = need_int(router, "experts", fw + "router: "), top = need_int(router, "top", fw + "router: ");
        if (top > experts) throw ConfigError("config.json: " + fw + "router: 'top' (" + std::to_string(top) + ") exceeds 'experts' (" + std::to_string(experts) + ")");
        Json ro = Json::object();
        ro.set("experts", experts);
        ro.set("top", top);
        fo.set("router", ro);
        fo.set("shared", given(*mlp, "shared") ? read_ff(mlp->at("shared"), fw + "shared: ") : Json());
      } else {
        throw ConfigError("config.json: " + fw + "'kind' = '" + kind + "' is not served (dense, moe)");
      }
      lo.set("mlp", fo);
    } else {
      lo.set("mlp", Json());
    }
    ls.push(lo);
  }
  out.set("layers", ls);
  return out;
}

ModelSpec lupolorn_spec(const Json& config) {
  const Json c = lupolorn_typed_config(config);
  const int64_t H = c.at("width").as_int(), V = c.at("vocab").as_int();
  const double eps = c.at("norm").at("eps").as_double();
  ModelSpec spec;
  spec.architecture = "Lupolorn";
  spec.vocab_size = V;
  spec.hidden_size = H;
  auto norm = [&](const std::string& tensor) {
    PartSpec p;
    p.kind = "rmsnorm";
    p.params.set("dim", H);
    p.params.set("eps", eps);
    p.params.set("tensor", tensor);
    return p;
  };
  auto two_layer = [&](int64_t ff) {      // W_down relu(W_up h)^2
    PartSpec p;
    p.kind = "dense";
    p.params.set("hidden", H);
    p.params.set("intermediate", ff);
    p.params.set("activation", "relu2");
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
    const std::string type = l.at("type").as_string();
    LayerSpec ls;
    ls.prefix = "l" + std::to_string(i);
    ls.block.kind = "sandwich";
    ls.block.params.set("defer_write", i + 1 < layers.size());      // the next layer's first read takes the last write in
    ls.parts.emplace_back("norm1", norm(ls.prefix + ".norm1"));
    PartSpec mix;
    mix.kind = type;
    mix.name = "mix";
    mix.params.set("hidden", H);
    const std::string at = ls.prefix + ".mix";
    if (type == "mingru") {
      mix.params.set("width", m.at("width").as_int());
    } else {
      mix.params.set("heads", m.at("heads").as_int());
      mix.params.set("head_dim", m.at("dim").as_int());
      mix.params.set("v_head_dim", m.at("vdim").as_int());
      mix.params.set("scale", m.at("scale").as_double());
      mix.params.set("eps", eps);
      if (type == "latent_attention") {
        mix.params.set("rot_dim", 0);
        mix.params.set("q_rank", m.at("q_rank").as_int());
        mix.params.set("kv_rank", m.at("kv_rank").as_int());
        mix.params.set("sink", false);
        if (m.has("mask")) mix.params.set("window", m.at("mask").at("size").as_int());
      } else {
        mix.params.set("kv_heads", m.at("kv_heads").as_int());
        mix.params.set("qk_norm", "unit_after");
        mix.params.set("sink_value", 0.0);
        mix.params.set("gate", "head");
        mix.params.set("gate_tensor", at + ".g");
        for (const char* t : {"q", "k", "v", "o"}) mix.params.set(t, at + "." + t);
        if (m.has("rot") && m.at("rot").at("dims").as_int() > 0) {
          const Json& rot = m.at("rot");
          PartSpec pos;
          pos.kind = "rope_partial";
          pos.params.set("dims", rot.at("dims").as_int());
          pos.params.set("base", rot.at("base").as_double());
          pos.params.set("layout", "pairs");
          if (rot.has("scaling")) {
            Json sc = rot.at("scaling");
            sc.set("kind", "wavelength");
            pos.params.set("scaling", sc);
          }
          mix.params.set("pos", pos.to_json());
        }
      }
    }
    ls.parts.emplace_back("mixer", mix);
    ls.parts.emplace_back("norm1b", norm(ls.prefix + ".norm1b"));
    if (l.has("mlp")) {
      const Json& f = l.at("mlp");
      ls.parts.emplace_back("norm2", norm(ls.prefix + ".norm2"));
      PartSpec ff;
      if (f.at("kind").as_string() == "dense") {
        ff = two_layer(f.at("ff").as_int());
      } else {
        ff.kind = "moe";
        ff.params.set("hidden", H);
        ff.params.set("intermediate", f.at("expert").at("ff").as_int());
        ff.params.set("experts", f.at("router").at("experts").as_int());
        ff.params.set("top", f.at("router").at("top").as_int());
        ff.params.set("activation", "relu2");
        ff.params.set("score", "softmax");
        ff.params.set("renormalize", false);
        ff.params.set("scale_input", false);
        if (f.has("shared")) {
          PartSpec sh = two_layer(f.at("shared").at("ff").as_int());
          sh.name = "shared";
          ff.params.set("shared", sh.to_json());
          ff.params.set("shared_gate", true);
          ff.params.set("shared_gate_tensor", ls.prefix + ".mlp.shared.sg");
        }
      }
      ff.name = "mlp";
      ls.parts.emplace_back("ffn", ff);
      ls.parts.emplace_back("norm2b", norm(ls.prefix + ".norm2b"));
    }
    if (!l.has("mlp")) {      // the norms around a feed-forward that is not there may lie in the checkpoint all the same
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
  spec.lm_head.params.set("tied", true);
  spec.lm_head.params.set("tied_to", "embed");
  return spec;
}

}  // namespace tinyinfer
