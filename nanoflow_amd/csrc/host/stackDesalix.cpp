// Desalix: a decoder with a norm on both sides of every sublayer (one number each) and a scale per column of what a
// sublayer adds, x += ls * rms(f(rms(x))); a run of its layers is passed several times with the same weights, the embedding
// output and a vector of the pass entering again.  Its mixer
//   attention   grouped-query attention within chunks of positions, a norm per head of q, k and v, rotate-half positions
//               on a part of q and k and on the whole of v (taken back from the output), a sink per head.
// The feed-forward is a mixture of clamped gated experts, chosen by their own sigmoids, which weigh the experts' inputs,
// beside one of the same form that every token has; a layer may have none.
#include <cmath>
#include <stdexcept>

#include "stackModel.h"

namespace {

using mini_json::Value;

constexpr double kGateSlope = 1.702, kUpShift = 1.0;

bool given(const Value& v, const char* key) { return v.contains(key) && !v.at(key).is_null(); }
int integer(const Value& v, const char* key) {
  const double x = v.at(key).number();
  if (x != std::floor(x) || std::fabs(x) > 1e9) throw std::runtime_error(std::string(key) + " must be an integer");
  return (int)x;
}

AttentionSpec attention(const Value& m) {
  AttentionSpec a;
  a.prefix = "mix.";
  a.heads = integer(m, "heads");
  a.kv_heads = integer(m, "kv_heads");
  a.dim = integer(m, "dim");
  a.vdim = integer(m, "vdim");
  a.scale = m.at("scale").number();
  if (given(m, "mask") && given(m.at("mask"), "size")) {
    a.chunk = integer(m.at("mask"), "size");
    if (a.chunk < 1) throw std::runtime_error("mask.size must be at least 1");
  }
  a.qk_norm = true;
  a.sink = true;
  a.value_norm = true;
  if (given(m, "rot")) {
    const Value& r = m.at("rot");
    a.rot = RotationSpec{integer(r, "dims"), r.at("base").number()};
    a.value_rot = RotationSpec{a.vdim, a.rot.base};
  }
  return a;
}

MixtureSpec mixture(const Value& f) {
  if (f.at("kind").str != "moe") throw std::runtime_error("unknown feed-forward \"" + f.at("kind").str + "\"");
  const Value &r = f.at("router"), &e = f.at("expert");
  MixtureSpec m;
  m.experts = integer(r, "experts");
  m.top = integer(r, "top");
  m.ff = integer(e, "ff");
  m.correction = false;
  m.scores = NF_SCORES_SIGMOID;
  m.weigh_input = true;
  m.shared_gate = false;
  m.gated = MixtureSpec::Gated{kGateSlope, kUpShift, e.at("limit").number(), 0};
  if (given(f, "shared")) {
    m.shared_ff = integer(f.at("shared"), "ff");
    m.gated->shared_limit = f.at("shared").at("limit").number();
  }
  return m;
}

StackModelSpec parse(const Value& c) {
  StackModelSpec s;
  s.width = integer(c, "width");
  s.vocab = integer(c, "vocab");
  s.eps = c.at("norm").at("eps").number();
  s.pre_norm = s.post_norm = true;
  s.scalar_norms = true;
  s.layer_scale = true;
  s.embedding_scale = c.at("embedding").at("scale").number();
  if (given(c, "loop")) {
    const Value& l = c.at("loop");
    s.loop = LoopSpec{integer(l, "start"), integer(l, "stop"), integer(l, "times")};
  }
  for (const Value& layer : c.at("layers").arr) {
    LayerSpec l;
    if (layer.at("type").str != "attention") throw std::runtime_error("unknown mixer \"" + layer.at("type").str + "\"");
    l.attention = attention(layer.at("mixer"));
    if (given(layer, "mlp")) l.mixture = mixture(layer.at("mlp"));
    s.layers.push_back(std::move(l));
  }
  return s;
}

const RegisterStackArchitecture registered("Desalix", parse);

}  // namespace
