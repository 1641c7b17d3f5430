// Pudadra: a pre-norm decoder (RMS norms whose weights are stored around zero, every sublayer added with the same
// multiplier, the embedding table read again as the output projection) whose layers have one of two mixers:
//   attention         differential attention over a window: two maps per head over the same values, q, k and v through a short
//                     convolution each, rotate-half positions with stretched wavelengths, capped scores, the maps'
//                     difference normed per head;
//   latent_attention  keys and values from one cached latent row per position, a rotated part shared by the heads, over a
//                     window.
// The feed-forward is dense (GELU) or a mixture of squared-ReLU experts chosen from the best groups, beside them a gated
// expert that every token has; a layer may have none.
#include <cmath>
#include <stdexcept>

#include "stackModel.h"

namespace {

using mini_json::Value;

bool given(const Value& v, const char* key) { return v.contains(key) && !v.at(key).is_null(); }
int integer(const Value& v, const char* key) {
  const double x = v.at(key).number();
  if (x != std::floor(x) || std::fabs(x) > 1e9) throw std::runtime_error(std::string(key) + " must be an integer");
  return (int)x;
}

RotationSpec rotation(const Value& m, bool interleaved) {
  RotationSpec r;
  if (!given(m, "rot")) return r;
  const Value& v = m.at("rot");
  r.dims = integer(v, "dims");
  r.base = v.at("base").number();
  r.interleaved = interleaved;
  if (given(v, "scaling")) {
    const Value& s = v.at("scaling");
    r.scaling = RotationScaling{s.at("factor").number(), s.at("low").number(), s.at("high").number(), s.at("original").number()};
  }
  return r;
}

int window(const Value& m) {  // 0: everything before
  if (!given(m, "mask") || !given(m.at("mask"), "size")) return 0;
  const int size = integer(m.at("mask"), "size");
  if (size < 1) throw std::runtime_error("mask.size must be at least 1");
  return size;
}

AttentionSpec attention(const Value& m) {
  AttentionSpec a;
  a.prefix = "mix.";
  a.heads = integer(m, "heads");
  a.kv_heads = integer(m, "kv_heads");
  a.dim = integer(m, "dim");
  a.vdim = integer(m, "vdim");
  a.scale = m.at("scale").number();
  if (given(m, "softcap")) a.softcap = m.at("softcap").number();
  a.window = window(m);
  a.rot = rotation(m, false);
  if (given(m, "conv")) a.conv_taps = integer(m, "conv");
  a.difference = m.at("diff").number();
  a.head_norm = true;
  a.out_scale = 1.0 - *a.difference;
  return a;
}

LatentAttentionSpec latent_attention(const Value& m) {
  LatentAttentionSpec a;
  a.prefix = "mix.";
  a.heads = integer(m, "heads");
  a.dim = integer(m, "dim");
  a.rot_dim = integer(m, "rot_dim");
  a.vdim = integer(m, "vdim");
  a.kv_rank = integer(m, "kv_rank");
  a.scale = m.at("scale").number();
  a.window = window(m);
  a.rot = rotation(m, true);
  return a;
}

MixtureSpec mixture(const Value& f) {
  const Value& r = f.at("router");
  MixtureSpec m;
  m.experts = integer(r, "experts");
  m.top = integer(r, "top");
  if (given(r, "groups")) {
    m.groups = integer(r.at("groups"), "count");
    m.keep_groups = integer(r.at("groups"), "keep");
  }
  m.correction = false;
  m.ff = integer(f.at("expert"), "ff");
  if (given(f, "shared")) m.shared_ff = integer(f.at("shared"), "ff");
  m.act = NF_ACT_SQUARED_RELU;
  return m;
}

StackModelSpec parse(const Value& c) {
  StackModelSpec s;
  s.width = integer(c, "width");
  s.vocab = integer(c, "vocab");
  s.eps = c.at("norm").at("eps").number();
  s.pre_norm = true;
  s.norm_offset = 1.0;
  s.residual_scale = c.at("residual_mult").number();
  s.logit_scale = c.at("logit_scale").number();
  s.tied_head = true;
  for (const Value& layer : c.at("layers").arr) {
    LayerSpec l;
    const std::string& type = layer.at("type").str;
    const Value& m = layer.at("mixer");
    if (type == "attention") l.attention = attention(m);
    else if (type == "latent_attention") l.latent = latent_attention(m);
    else throw std::runtime_error("unknown mixer \"" + type + "\"");
    if (given(layer, "mlp")) {
      const Value& f = layer.at("mlp");
      const std::string& kind = f.at("kind").str;
      if (kind == "dense") l.mlp = MlpSpec{integer(f, "ff"), NF_ACT_GELU};
      else if (kind == "moe") l.mixture = mixture(f);
      else throw std::runtime_error("unknown feed-forward \"" + kind + "\"");
    }
    s.layers.push_back(std::move(l));
  }
  return s;
}

const RegisterStackArchitecture registered("Pudadra", parse);

}  // namespace
