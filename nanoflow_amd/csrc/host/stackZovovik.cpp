// Zovovik: a decoder with learned positions whose layers are norm-on-output sublayers
// (x += norm(mixer(x)), x += norm(ff(x))) with one of two mixers:
//   retention  a fixed decay per head, rotate-half positions on q and k;
//   parallel   left: attention over a window with kept first positions, per-head q / k norm, interleaved
//              rotation and a sink per head; right: a recurrence with data-dependent decay on
//              token-shifted inputs; the two outputs are added with a scale each.
// The feed-forward is dense with a squared ReLU; a layer may have none.
#include <stdexcept>

#include "stackModel.h"

namespace {

using mini_json::Value;

int integer(const Value& v, const char* key) { return (int)v.at(key).number(); }

RotationSpec rotation(const Value& mixer, bool interleaved) {
  const Value& r = mixer.at("rot");
  return RotationSpec{integer(r, "dims"), r.at("base").number(), interleaved};
}

RecurrenceSpec retention(const Value& m) {
  RecurrenceSpec r;
  r.prefix = "mix.";
  r.kind = NF_RECURRENCE_FIXED_DECAY;
  r.heads = integer(m, "heads");
  r.dim = integer(m, "dim");
  r.vdim = integer(m, "vdim");
  for (const Value& d : m.at("decay").arr) r.decay.push_back(d.number());
  r.rot = rotation(m, false);
  r.k_scale = 1.0 / __builtin_sqrt((double)r.dim);
  return r;
}

AttentionSpec window_attention(const Value& m, double out_scale) {
  AttentionSpec a;
  a.prefix = "mix.left.";
  a.heads = integer(m, "heads");
  a.kv_heads = integer(m, "kv_heads");
  a.dim = integer(m, "dim");
  a.vdim = integer(m, "vdim");
  a.scale = m.at("scale").number();
  a.window = integer(m.at("mask"), "size");
  a.keep_first = integer(m.at("mask"), "keep_first");
  if (a.window < 1) throw std::runtime_error("mask.size must be at least 1");
  a.qk_norm = true;
  a.sink = true;
  a.rot = rotation(m, true);
  a.out_scale = out_scale;
  return a;
}

RecurrenceSpec token_shift(const Value& m, double out_scale) {
  RecurrenceSpec r;
  r.prefix = "mix.right.";
  r.kind = NF_RECURRENCE_TOKEN_DECAY;
  r.heads = integer(m, "heads");
  r.dim = r.vdim = integer(m, "dim");
  r.out_scale = out_scale;
  return r;
}

StackModelSpec parse(const Value& c) {
  StackModelSpec s;
  s.width = integer(c, "width");
  s.vocab = integer(c, "vocab");
  s.max_positions = integer(c, "max_positions");
  s.eps = c.at("norm").at("eps").number();
  s.learned_positions = true;
  for (const Value& layer : c.at("layers").arr) {
    LayerSpec l;
    const std::string& type = layer.at("type").str;
    const Value& m = layer.at("mixer");
    if (type == "retention") {
      l.recurrence = retention(m);
    } else if (type == "parallel") {
      l.attention = window_attention(m.at("left"), m.at("left_scale").number());
      l.recurrence = token_shift(m.at("right"), m.at("right_scale").number());
    } else {
      throw std::runtime_error("unknown mixer \"" + type + "\"");
    }
    if (layer.contains("mlp") && !layer.at("mlp").is_null()) {
      const Value& f = layer.at("mlp");
      if (f.at("kind").str != "dense") throw std::runtime_error("unknown feed-forward \"" + f.at("kind").str + "\"");
      l.mlp = MlpSpec{integer(f, "ff"), NF_ACT_SQUARED_RELU};
    }
    s.layers.push_back(std::move(l));
  }
  return s;
}

const RegisterStackArchitecture registered("Zovovik", parse);

}  // namespace
