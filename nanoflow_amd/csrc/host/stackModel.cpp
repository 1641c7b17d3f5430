#include "stackModel.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>
#include <cstring>
#include <stdexcept>

#include "helper.h"
#include "operatorWrapper.h"

std::shared_ptr<StackModelConfig> ActiveStackModel;

std::map<std::string, StackParser>& stackArchitectures() {
  static std::map<std::string, StackParser> m;
  return m;
}

StackModelSpec parseStackModel(const mini_json::Value& config) {
  if (!config.contains("architecture")) throw std::runtime_error("the model configuration names no architecture");
  const std::string& name = config.at("architecture").str;
  auto it = stackArchitectures().find(name);
  if (it == stackArchitectures().end()) throw std::runtime_error("unknown architecture \"" + name + "\"");
  StackModelSpec s = it->second(config);
  s.architecture = name;
  auto require = [&](bool ok, const std::string& what) {
    if (!ok) throw std::runtime_error(name + ": " + what);
  };
  require(s.width > 0 && s.vocab > 0 && s.max_positions >= 0 && !s.layers.empty(), "width, vocab and layers must be positive");
  require(s.max_positions > 0 || !s.learned_positions, "max_positions must be positive");
  require(s.token_side >= 0, "the token input's size");
  require(!s.post_norm || s.pre_norm, "norms on both sides of a sublayer");
  require(!s.layer_scale || s.post_norm || !s.pre_norm, "a scale per column goes with a norm of the sublayer's output");
  require(!s.loop || (s.loop->start >= 0 && s.loop->start < s.loop->stop && s.loop->stop <= (int)s.layers.size() && s.loop->times > 0 &&
                      (long long)(s.loop->stop - s.loop->start) * s.loop->times <= 100000),
          "loop.start < loop.stop among the layers, loop.times at least 1");
  for (size_t i = 0; i < s.layers.size(); ++i) {
    const LayerSpec& l = s.layers[i];
    const std::string at = "layer " + std::to_string(i) + ": ";
    require(l.attention || l.recurrence || l.latent, at + "no mixer");
    require(!l.latent || (!l.attention && !l.recurrence), at + "latent attention beside another mixer");
    require(!l.mlp || !l.mixture, at + "two feed-forwards");
    auto rotation = [&](const RotationSpec& r, int dim) {
      require(r.dims >= 0 && r.dims <= dim && r.dims % 2 == 0, at + "rotated dimensions");
      require(!r.scaling || (r.scaling->factor > 0 && r.scaling->low > 0 && r.scaling->high > r.scaling->low && r.scaling->original > 0),
              at + "scaling of the rotation");
    };
    if (l.attention) {
      const auto& a = *l.attention;
      require(a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0, at + "query heads must be a multiple of the kv heads");
      require(a.dim > 0 && a.dim <= 256 && a.vdim > 0 && a.vdim <= 256, at + "attention head sizes must be in 1..256");
      rotation(a.rot, a.dim);
      require(a.window >= 0 && a.keep_first >= 0 && a.chunk >= 0, at + "window");
      rotation(a.value_rot, a.vdim);
      require(!a.value_rot.scaling && (a.value_rot.dims == 0 || a.value_rot.dims == a.vdim), at + "rotated values");
      require(a.value_rot.dims == 0 || (a.conv_taps == 0 && !a.bias), at + "rotated values of a biased or convolved projection");
      require(!a.q_temp || a.q_temp->every > 0, at + "query temperature");
      require(!a.sink || !a.unit_sink, at + "two sinks");
      require(!a.difference || (!a.sink && !a.unit_sink), at + "a sink in a difference of attentions");
      require(a.softcap >= 0, at + "bound of the scores");
      require(a.conv_taps >= 0 && a.conv_taps <= 64, at + "a convolution has 1..64 taps");
    }
    if (l.latent) {
      const auto& a = *l.latent;
      require(a.heads > 0 && a.dim > 0 && a.vdim > 0 && a.rot_dim >= 0 && a.rot_dim <= 256 && a.kv_rank > 0 && a.kv_rank <= 2048,
              at + "latent attention sizes (a latent of 1..2048, a rotated part of 0..256)");
      require(a.window >= 0, at + "window");
      rotation(a.rot, a.rot_dim);
    }
    if (l.recurrence) {
      const auto& r = *l.recurrence;
      require(r.heads > 0 && r.dim > 0 && r.dim <= 256 && r.vdim > 0 && r.vdim <= 256, at + "recurrence head sizes must be in 1..256");
      rotation(r.rot, r.dim);
      require(r.kind != NF_RECURRENCE_TOKEN_DECAY || !s.pre_norm, at + "a token shift reads the residual stream itself, not its norm");
      require(r.kind == NF_RECURRENCE_FIXED_DECAY || (!r.joint_norm && r.qkv_act == NF_ACT_NONE), at + "projections of a fixed-decay recurrence only");
      require(r.kind != NF_RECURRENCE_FIXED_DECAY || (int)r.decay.size() == r.heads, at + "one decay per head");
    }
    if (l.mlp) require(l.mlp->ff > 0, at + "feed-forward width");
    if (l.mixture) {
      const auto& m = *l.mixture;
      require(m.ff > 0, at + "feed-forward width");
      require(m.experts > 0 && m.identity >= 0 && m.experts + m.identity <= 1024, at + "1..1024 experts, the identity experts among them");
      require(m.top > 0 && m.top <= m.experts + m.identity && m.top <= 64, at + "a token uses 1..64 of the experts");
      require(!m.weigh_input || m.identity == 0, at + "identity experts with a weighed input");
      require(!m.gated || (m.gated->limit >= 0 && m.gated->shared_limit >= 0), at + "limit of the experts");
      require(m.groups > 0 && m.outputs() % m.groups == 0 && m.keep_groups > 0 && m.keep_groups <= m.groups &&
                  m.top <= m.outputs() / m.groups * m.keep_groups,
              at + "equal groups of experts, the kept ones with room for the choice");
      require(m.shared_ff >= 0 && (m.shared_ff == 0 || m.always() > 0), at + "a shared expert beside at most 63 chosen ones");
    }
  }
  return s;
}

std::vector<LayerRun> StackModelSpec::runs() const {
  std::vector<LayerRun> r;
  const LoopSpec l = loop ? *loop : LoopSpec{0, 0, 0};
  for (int i = 0; i < l.start; ++i) r.push_back({i, -1});
  for (int t = 0; t < l.times; ++t)
    for (int i = l.start; i < l.stop; ++i) r.push_back({i, i == l.start ? t : -1});
  for (int i = l.stop; i < (int)layers.size(); ++i) r.push_back({i, -1});
  return r;
}

// ---------------------------------------------------------------- safetensors
SafetensorsFile::SafetensorsFile(const std::string& path) {
  const int fd = ::open(path.c_str(), O_RDONLY);
  if (fd < 0) throw std::runtime_error("cannot open " + path);
  struct stat st;
  if (::fstat(fd, &st) != 0 || st.st_size < 8) {
    ::close(fd);
    throw std::runtime_error(path + ": too short for a safetensors file");
  }
  bytes_ = (size_t)st.st_size;
  map_ = ::mmap(nullptr, bytes_, PROT_READ, MAP_PRIVATE, fd, 0);
  ::close(fd);
  if (map_ == MAP_FAILED) {
    map_ = nullptr;
    throw std::runtime_error("cannot map " + path);
  }
  try {
    const uint8_t* p = static_cast<const uint8_t*>(map_);
    uint64_t n = 0;
    for (int i = 7; i >= 0; --i) n = n << 8 | p[i];
    if (n > bytes_ - 8) throw std::runtime_error(path + ": header length beyond the file");
    const std::string header(reinterpret_cast<const char*>(p) + 8, (size_t)n);
    const mini_json::Value j = mini_json::Parser(header).parse();
    const size_t base = 8 + (size_t)n;
    for (const auto& [name, v] : j.obj) {
      if (name == "__metadata__") continue;
      HostTensor t;
      const std::string& type = v.at("dtype").str;
      if (type == "BF16") t.type = HostTensor::BF16;
      else if (type == "F32") t.type = HostTensor::F32;
      else if (type == "I32") t.type = HostTensor::I32;
      else throw std::runtime_error(path + ": tensor " + name + " has type " + type);
      for (const auto& d : v.at("shape").arr) t.shape.push_back((int64_t)d.number());
      const auto& off = v.at("data_offsets").arr;
      if (off.size() != 2) throw std::runtime_error(path + ": tensor " + name + " has no data_offsets");
      const size_t from = (size_t)off[0].number(), to = (size_t)off[1].number();
      if (from > to || to > bytes_ - base || to - from != t.elements() * (t.type == HostTensor::BF16 ? 2 : 4))
        throw std::runtime_error(path + ": tensor " + name + " does not fit its data_offsets");
      t.data = p + base + from;
      tensors_[name] = t;
    }
  } catch (...) {
    ::munmap(map_, bytes_);
    map_ = nullptr;
    throw;
  }
}

SafetensorsFile::~SafetensorsFile() {
  if (map_) ::munmap(map_, bytes_);
}

// ---------------------------------------------------------------- upload
static float bf16_to_float(uint16_t b) {
  const uint32_t u = (uint32_t)b << 16;
  float f;
  std::memcpy(&f, &u, 4);
  return f;
}
static uint16_t float_to_bf16(float f) {  // round to nearest even
  uint32_t u;
  std::memcpy(&u, &f, 4);
  if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40);
  return (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
}
static float element(const HostTensor& t, size_t i) {
  if (t.type == HostTensor::BF16) {
    uint16_t b;
    std::memcpy(&b, static_cast<const uint8_t*>(t.data) + 2 * i, 2);
    return bf16_to_float(b);
  }
  if (t.type == HostTensor::F32) {
    float f;
    std::memcpy(&f, static_cast<const uint8_t*>(t.data) + 4 * i, 4);
    return f;
  }
  int32_t v;
  std::memcpy(&v, static_cast<const uint8_t*>(t.data) + 4 * i, 4);
  return (float)v;
}
static int pad8(int n) { return (n + 7) / 8 * 8; }

struct StackModel::Loader {
  StackModel& m;
  const HostTensors& tensors;
  std::vector<uint8_t> staging;

  const HostTensor& get(const std::string& name, std::vector<int64_t> shape) {
    auto it = tensors.find(name);
    if (it == tensors.end()) throw std::runtime_error("tensor " + name + " is missing");
    if (it->second.shape != shape) {
      std::string want, have;
      for (auto d : shape) want += " " + std::to_string(d);
      for (auto d : it->second.shape) have += " " + std::to_string(d);
      throw std::runtime_error("tensor " + name + " has shape" + have + ", the configuration asks for" + want);
    }
    return it->second;
  }
  // rows of several [n_i][k] tensors, one below the other
  // halves > 0: in groups of `halves` rows (columns of an output projection), row c of a group's first half and row
  // c of its second are laid beside each other -- pairs of a rotation by halves, for operators that turn neighbours
  struct Part {
    std::string name;
    int rows;
    int halves = 0;
    int place(int i) const {
      if (halves == 0) return i;
      const int c = i % halves, half = halves / 2;
      return i - c + (c < half ? 2 * c : 2 * (c - half) + 1);
    }
  };
  void put(uint8_t* dst, float f) {
    if (m.dtype == NF_BF16) {
      const uint16_t b = float_to_bf16(f);
      std::memcpy(dst, &b, 2);
    } else {
      std::memcpy(dst, &f, 4);
    }
  }
  // rows [from_row, + rows), columns [from_col, + cols) of a tensor whose rows have `t_cols`, to (row0, col0)
  void put_block(const HostTensor& t, int t_cols, int from_row, int rows, int from_col, int cols, int row0, int col0, int K) {
    const size_t es = m.elementBytes();
    for (int r = 0; r < rows; ++r) {
      uint8_t* dst = staging.data() + ((size_t)(row0 + r) * K + col0) * es;
      const size_t src = (size_t)(from_row + r) * t_cols + from_col;
      if (m.dtype == NF_BF16 && t.type == HostTensor::BF16)
        std::memcpy(dst, static_cast<const uint8_t*>(t.data) + src * 2, (size_t)cols * 2);
      else
        for (int c = 0; c < cols; ++c) put(dst + es * c, element(t, src + c));
    }
  }
  void put_rows(const HostTensor& t, int rows, int cols, int row0, int col0, int K) { put_block(t, cols, 0, rows, 0, cols, row0, col0, K); }
  void start(size_t N, size_t K) { staging.assign(N * K * m.elementBytes(), 0); }
  DeviceMatrix finish(int N, int K) {
    DeviceMatrix d;
    d.N = N;
    d.K = K;
    d.ptr = m.allocate(staging.size());
    HIP_CHECK(hipMemcpy(d.ptr, staging.data(), staging.size(), hipMemcpyHostToDevice));
    return d;
  }
  DeviceMatrix matrix(const std::vector<Part>& parts, int cols, std::vector<int>* first_row = nullptr) {
    int rows = 0;
    for (const auto& p : parts) rows += p.rows;
    const int N = pad8(rows), K = pad8(cols);
    start(N, K);
    int at = 0;
    for (const auto& p : parts) {
      if (first_row) first_row->push_back(at);
      const HostTensor& t = get(p.name, {p.rows, cols});
      if (p.halves == 0) put_rows(t, p.rows, cols, at, 0, K);
      else for (int r = 0; r < p.rows; ++r) put_block(t, cols, r, 1, 0, cols, at + p.place(r), 0, K);
      at += p.rows;
    }
    return finish(N, K);
  }
  // [rows][k_1 | k_2 | ...]: output projections of mixers side by side, applied to their concatenated heads
  DeviceMatrix columns(const std::vector<Part>& parts, int rows) {
    int cols = 0;
    for (const auto& p : parts) cols += p.rows;
    const int N = pad8(rows), K = pad8(cols);
    start(N, K);
    int at = 0;
    for (const auto& p : parts) {
      const HostTensor& t = get(p.name, {rows, p.rows});
      if (p.halves == 0) put_rows(t, rows, p.rows, 0, at, K);
      else for (int c = 0; c < p.rows; ++c) put_block(t, p.rows, 0, rows, c, 1, 0, at + p.place(c), K);
      at += p.rows;
    }
    return finish(N, K);
  }
  // one row of N elements: the tensors of `parts` (1-d) at the places given
  void* row(const std::vector<Part>& parts, const std::vector<int>& at, int N) {
    start(1, N);
    for (size_t i = 0; i < parts.size(); ++i) put_rows(get(parts[i].name, {parts[i].rows}), 1, parts[i].rows, 0, at[i], N);
    return finish(1, N).ptr;
  }
  // `columns`: a tensor that multiplies the weights column by column
  nf_norm norm(const std::string& name, nf_norm_kind kind, double scale = 1, const std::string& columns = "") {
    const int W = m.spec.width, ld = m.spec.ld();
    if (m.spec.scalar_norms || !columns.empty()) {
      std::vector<float> v((size_t)ld, 0.f);
      const HostTensor& w = m.spec.scalar_norms ? get(name, {}) : get(name, {W});
      const HostTensor* by = columns.empty() ? nullptr : &get(columns, {W});
      for (int c = 0; c < W; ++c)
        v[c] = (float)((element(w, m.spec.scalar_norms ? 0 : c) + m.spec.norm_offset) * scale * (by ? element(*by, c) : 1.0));
      return nf_norm{kind, upload(v), kind == NF_NORM_LAYER ? vectors({name + ".b"}, {W}, W, ld) : nullptr, (float)m.spec.eps};
    }
    return nf_norm{kind, vectors({name}, {W}, W, ld, m.spec.norm_offset, scale), kind == NF_NORM_LAYER ? vectors({name + ".b"}, {W}, W, ld) : nullptr, (float)m.spec.eps};
  }

  void latent(const LatentAttentionSpec& a, const std::string& p, LayerWeights& lw) {
    LatentAttentionWeights& w = lw.latent;
    const int W = m.spec.width, K = pad8(W), H = a.heads, R = a.kv_rank, rp = pad8(R);
    const int dp = w.dim_pad = pad8(a.dim), vp = w.vdim_pad = pad8(a.vdim), head = a.dim + a.rot_dim;
    w.q_col = H * dp;
    w.kv_col = w.q_col + H * a.rot_dim;
    const int N = pad8(w.kv_col + R + a.rot_dim);
    start(N, K);
    const HostTensor& q = get(p + "q", {H * head, W});
    for (int h = 0; h < H; ++h) {
      put_block(q, W, h * head, a.dim, 0, W, h * dp, 0, K);
      put_block(q, W, h * head + a.dim, a.rot_dim, 0, W, w.q_col + h * a.rot_dim, 0, K);
    }
    put_rows(get(p + "dkv", {R + a.rot_dim, W}), R + a.rot_dim, W, w.kv_col, 0, K);
    w.proj = finish(N, K);
    w.norm = vectors({p + "dkv.norm"}, {R}, R, rp);
    const HostTensor& uk = get(p + "uk", {H * a.dim, R});
    start((size_t)H * rp, dp);
    for (int h = 0; h < H; ++h)
      for (int c = 0; c < R; ++c)
        for (int d = 0; d < a.dim; ++d)
          put(staging.data() + (((size_t)h * rp + c) * dp + d) * m.elementBytes(), element(uk, (size_t)(h * a.dim + d) * R + c));
    w.to_latent = finish(rp, dp);
    const HostTensor& uv = get(p + "uv", {H * a.vdim, R});
    start((size_t)H * (dp + vp), rp);
    for (int h = 0; h < H; ++h) {
      put_block(uk, R, h * a.dim, a.dim, 0, R, h * dp, 0, rp);
      put_block(uv, R, h * a.vdim, a.vdim, 0, R, H * dp + h * vp, 0, rp);
    }
    w.expand = finish(H * (dp + vp), rp);
    w.from_latent = DeviceMatrix{(uint8_t*)w.expand.ptr + (size_t)H * dp * rp * m.elementBytes(), vp, rp};
    const HostTensor& o = get(p + "o", {W, H * a.vdim});
    const int N_out = pad8(W), K_out = H * vp;
    start(N_out, K_out);
    for (int h = 0; h < H; ++h) put_block(o, H * a.vdim, 0, W, h * a.vdim, a.vdim, 0, h * vp, K_out);
    lw.out = finish(N_out, K_out);
    w.rot = m.rotation(a.rot);
  }

  void mixture(const MixtureSpec& s, const std::string& p, LayerWeights& w) {
    const int W = m.spec.width, columns = s.expertFf(), ff = pad8(columns), K = pad8(W), all = s.experts + s.always();
    auto share = [&](int j) { return std::max(0, std::min(columns, s.shared_ff - j * columns)); };  // of the shared expert's columns
    // gate and up: a column's two rows beside each other
    const std::vector<std::string> first = s.gated ? std::vector<std::string>{"gate", "up"} : std::vector<std::string>{"up"};
    const int n = (int)first.size();
    start((size_t)all * n * ff, K);
    for (int i = 0; i < n; ++i) {
      auto rows = [&](const HostTensor& t, int from, int count, int expert) {
        for (int r = 0; r < count; ++r) put_block(t, W, from + r, 1, 0, W, (expert * ff + r) * n + i, 0, K);
      };
      for (int e = 0; e < s.experts; ++e) rows(get(p + "e" + std::to_string(e) + "." + first[i], {s.ff, W}), 0, s.ff, e);
      for (int j = 0; j < s.always(); ++j) rows(get(p + "shared." + first[i], {s.shared_ff, W}), j * columns, share(j), s.experts + j);
    }
    w.up = finish(n * ff, K);
    start((size_t)all * K, ff);
    for (int e = 0; e < s.experts; ++e) put_rows(get(p + "e" + std::to_string(e) + ".down", {W, s.ff}), W, s.ff, e * K, 0, ff);
    for (int j = 0; j < s.always(); ++j)
      put_block(get(p + "shared.down", {W, s.shared_ff}), s.shared_ff, 0, W, j * columns, share(j), (s.experts + j) * K, 0, ff);
    w.down = finish(K, ff);
    std::vector<Part> router{{p + "router", s.outputs()}};
    if (s.always() > 0 && s.shared_gate) router.push_back({p + "shared.sg", 1});
    w.router = matrix(router, W);
    if (s.gated) {
      std::vector<float> limits((size_t)all, (float)s.gated->limit);
      for (int j = 0; j < s.always(); ++j) limits[s.experts + j] = (float)s.gated->shared_limit;
      w.limits = upload(limits);
    }
    if (s.correction) w.correction = vectors({p + "correction"}, {s.outputs()}, s.outputs(), s.outputs());
  }
  // weights [channels][taps] of convolutions on the columns from at[i] on -> [taps][N] in the activations' type
  void* taps(const std::vector<Part>& parts, const std::vector<int>& at, int n, int N) {
    start(n, N);
    for (size_t i = 0; i < parts.size(); ++i) {
      const HostTensor& t = get(parts[i].name, {parts[i].rows, n});
      for (int c = 0; c < parts[i].rows; ++c)
        for (int j = 0; j < n; ++j) put(staging.data() + ((size_t)j * N + at[i] + c) * m.elementBytes(), element(t, (size_t)c * n + j));
    }
    return finish(n, N).ptr;
  }
  // exp(lq1 . lk1) - exp(lq2 . lk2) + difference
  float map_weight(const AttentionSpec& a, const std::string& p) {
    auto dot = [&](const char* q, const char* k) {
      const HostTensor &x = get(p + q, {a.dim}), &y = get(p + k, {a.dim});
      double sum = 0;
      for (int c = 0; c < a.dim; ++c) sum += (double)element(x, c) * element(y, c);
      return sum;
    };
    return (float)(std::exp(dot("lq1", "lk1")) - std::exp(dot("lq2", "lk2")) + *a.difference);
  }
  float* upload(const std::vector<float>& v) {
    float* d = static_cast<float*>(m.allocate(v.size() * sizeof(float)));
    HIP_CHECK(hipMemcpy(d, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
    return d;
  }
  // vectors of `rows` x `cols`, each row padded to `ld`
  float* vectors(const std::vector<std::string>& names, std::vector<int64_t> shape, int cols, int ld, double offset = 0, double scale = 1) {
    std::vector<float> v((size_t)names.size() * ld, 0.f);
    for (size_t s = 0; s < names.size(); ++s) {
      const HostTensor& t = get(names[s], shape);
      for (int c = 0; c < cols; ++c) v[s * ld + c] = (float)((element(t, c) + offset) * scale);
    }
    return upload(v);
  }
};

void* StackModel::allocate(size_t bytes) {
  void* p = nullptr;
  bytes = std::max<size_t>((bytes + 255) / 256 * 256, 256);
  HIP_CHECK(hipMalloc(&p, bytes));
  HIP_CHECK(hipMemset(p, 0, bytes));
  owned_.push_back(p);
  return p;
}

double RotationSpec::frequency(int pair) const {
  const double f = std::pow(base, -2.0 * pair / dims);
  if (!scaling) return f;
  const double periods = scaling->original * f / (2 * M_PI);  // that fit into the original positions
  if (periods > scaling->high) return f;
  if (periods < scaling->low) return f / scaling->factor;
  const double s = (periods - scaling->low) / (scaling->high - scaling->low);
  return (1 - s) * f / scaling->factor + s * f;
}

// cos and sin of position * frequency, evaluated in double and kept in fp32: one table per distinct
// rotation, for every position a request can have.
nf_rotation StackModel::rotation(const RotationSpec& r) {
  nf_rotation out{nullptr, r.dims, r.interleaved ? 1 : 0};
  if (r.dims == 0) return out;
  std::vector<double> key{(double)r.dims, r.base};
  if (r.scaling) key.insert(key.end(), {r.scaling->factor, r.scaling->low, r.scaling->high, r.scaling->original});
  float*& table = rotation_tables_[key];
  if (!table) {
    const int half = r.dims / 2;
    std::vector<float> v((size_t)spec.max_positions * half * 2);
    for (int i = 0; i < half; ++i) {
      const double f = r.frequency(i);
      for (int p = 0; p < spec.max_positions; ++p) {
        v[((size_t)p * half + i) * 2] = (float)std::cos(p * f);
        v[((size_t)p * half + i) * 2 + 1] = (float)std::sin(p * f);
      }
    }
    table = static_cast<float*>(allocate(v.size() * sizeof(float)));
    HIP_CHECK(hipMemcpy(table, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
  }
  out.table = table;
  return out;
}

nf_latent_layout StackModel::latentLayout(int layer) const {
  const LatentAttentionSpec& a = *spec.layers[layer].latent;
  nf_latent_layout l{};
  NF_KERNEL_CHECK(nf_latent_layout_of(dtype, a.heads, a.kv_rank, a.rot_dim, page_size, &l));
  return l;
}

nf_kv_layout StackModel::expandedLayout(int layer) const {
  const LatentAttentionSpec& a = *spec.layers[layer].latent;
  const int dim = pad8(a.dim) + a.rot_dim, vdim = pad8(a.vdim);
  if (dtype != NF_BF16 || dim > 256 || vdim > 256) return nf_kv_layout{};
  return nf_kv_layout{dtype, a.heads, a.heads, dim, vdim, (dim + 31) / 32 * 32, (vdim + 15) / 16 * 16, page_size, 1};
}

nf_kv_layout StackModel::kvLayout(int layer) const {
  const AttentionSpec& a = *spec.layers[layer].attention;
  return nf_kv_layout{dtype, a.heads, a.kv_heads, a.dim, a.vdim, (a.dim + 31) / 32 * 32, (a.vdim + 15) / 16 * 16, page_size, a.maps()};
}

// Values that are turned by halves are kept with their pairs side by side: the value projection's rows and the output
// projection's columns are laid out for it.
static int halves_of_values(const AttentionSpec& a) { return a.value_rot.dims > 0 && !a.value_rot.interleaved ? a.vdim : 0; }

StackModel::StackModel(const StackModelSpec& spec_, const HostTensors& tensors, nf_dtype dtype_, int kv_pages_, int page_size_,
                       int state_slots_)
    : spec(spec_), dtype(dtype_), kv_pages(kv_pages_), page_size(page_size_), state_slots(state_slots_), runs(spec_.runs()) {
  const int W = spec.width, ld = spec.ld();
  Loader L{*this, tensors, {}};
  try {
    weights.embed = L.matrix({{"embed", spec.vocab}}, W);
    if (spec.learned_positions) weights.pos = L.matrix({{"pos", spec.max_positions}}, W);
    weights.head = spec.tied_head ? weights.embed : L.matrix({{"head", spec.vocab}}, W);
    // the logits' scale is one of the rows that the output projection reads
    weights.final_norm = L.norm("final.norm", spec.norm, spec.logit_scale);
    if (spec.token_side > 0) weights.side_embed = L.matrix({{"side.embed", spec.vocab}}, spec.token_side * (int)spec.layers.size());
    const int n = (int)spec.layers.size();
    weights.layers.resize(n);
    if (spec.loop) {
      const HostTensor& steps = L.get("loop.step", {spec.loop->times, W});
      std::vector<float> v((size_t)spec.loop->times * ld, 0.f);
      for (int t = 0; t < spec.loop->times; ++t)
        for (int c = 0; c < W; ++c) v[(size_t)t * ld + c] = element(steps, (size_t)t * W + c);
      weights.loop_step = L.upload(v);
    }
    kv_data.assign(runs.size(), nullptr);
    state.assign(runs.size(), nullptr);
    shift_state.assign(runs.size(), nullptr);
    conv_state.assign(runs.size(), nullptr);
    for (int i = 0; i < n; ++i) {
      const LayerSpec& s = spec.layers[i];
      LayerWeights& w = weights.layers[i];
      const std::string l = "l" + std::to_string(i) + ".";
      std::vector<Loader::Part> out_parts;
      if (s.attention) {
        const AttentionSpec& a = *s.attention;
        const std::string p = l + a.prefix;
        std::vector<int> at;
        std::vector<Loader::Part> parts{
            {p + "q", a.heads * a.maps() * a.dim}, {p + "k", a.kv_heads * a.maps() * a.dim}, {p + "v", a.kv_heads * a.vdim, halves_of_values(a)}};
        if (a.head_gate) parts.push_back({p + "g", a.heads});
        w.attention.qkv = L.matrix(parts, W, &at);
        if (a.head_gate) w.attention.g_col = at[3];
        if (a.bias)
          w.attention.bias = L.row({{p + "q.b", parts[0].rows}, {p + "k.b", parts[1].rows}, {p + "v.b", parts[2].rows}}, at, w.attention.qkv.N);
        w.attention.q_col = at[0];
        w.attention.k_col = at[1];
        w.attention.v_col = at[2];
        if (a.qk_norm) {
          w.attention.q_norm = L.vectors({p + "q.norm"}, {a.dim}, a.dim, a.dim);
          w.attention.k_norm = L.vectors({p + "k.norm"}, {a.dim}, a.dim, a.dim);
        }
        if (a.sink) w.attention.sink = L.vectors({p + "sink"}, {a.heads}, a.heads, a.heads);
        if (a.unit_sink) w.attention.sink = L.upload(std::vector<float>((size_t)a.heads, 0.f));
        if (a.difference) w.attention.map_weight = L.map_weight(a, p);
        if (a.conv_taps > 0) {
          w.attention.conv = L.taps({{p + "q.conv", parts[0].rows}, {p + "k.conv", parts[1].rows}, {p + "v.conv", parts[2].rows}}, at,
                                    a.conv_taps, w.attention.qkv.N);
        }
        w.attention.rot = rotation(a.rot);
        RotationSpec turned = a.value_rot;
        turned.interleaved = true;
        w.attention.value_rot = rotation(turned);
        out_parts.push_back({p + "o", a.heads * a.vdim, halves_of_values(a)});
      }
      if (s.recurrence) {
        const RecurrenceSpec& r = *s.recurrence;
        const std::string p = l + r.prefix;
        const int qk = r.heads * r.dim, vg = r.heads * r.vdim;
        if (r.kind == NF_RECURRENCE_FIXED_DECAY) {
          std::vector<int> at;
          std::vector<Loader::Part> parts{{p + "q", qk}, {p + "k", qk}, {p + "v", vg}};
          const bool g_apart = r.qkv_act != NF_ACT_NONE;
          if (!g_apart) parts.push_back({p + "g", vg});
          w.recurrence.qkvg = L.matrix(parts, W, &at);
          if (g_apart) w.recurrence.g = L.matrix({{p + "g", vg}}, W);
          if (r.joint_norm) w.recurrence.norm = L.vectors({p + "norm"}, {vg}, vg, pad8(vg));
          w.recurrence.q_col = at[0];
          w.recurrence.k_col = at[1];
          w.recurrence.v_col = at[2];
          w.recurrence.g_col = g_apart ? 0 : at[3];
          std::vector<float> d;
          for (double x : r.decay) d.push_back(x > 0 ? std::max((float)std::log2(x), -126.f) : -126.f);
          w.recurrence.log2_decay = L.upload(d);
          w.recurrence.rot = rotation(r.rot);
        } else {
          w.recurrence.r = L.matrix({{p + "r", qk}}, W);
          w.recurrence.k = L.matrix({{p + "k", qk}}, W);
          w.recurrence.v = L.matrix({{p + "v", vg}}, W);
          w.recurrence.g = L.matrix({{p + "g", vg}}, W);
          auto it = tensors.find(p + "w1");  // the rank of the decay's two-step projection is the tensor's own
          if (it == tensors.end() || it->second.shape.size() != 2) throw std::runtime_error("tensor " + p + "w1 is missing");
          const int rank = (int)it->second.shape[0];
          w.recurrence.w1 = L.matrix({{p + "w1", rank}}, W);
          w.recurrence.w2 = L.matrix({{p + "w2", qk}}, rank);
          w.recurrence.w0 = L.vectors({p + "w0"}, {qk}, qk, pad8(qk));
          w.recurrence.u = L.vectors({p + "u"}, {r.heads, r.dim}, qk, qk);
          w.recurrence.norm = L.vectors({p + "norm"}, {vg}, vg, vg);
          w.recurrence.mu = L.vectors({p + "mu.r", p + "mu.k", p + "mu.v", p + "mu.g", p + "mu.w"}, {W}, W, ld);
        }
        out_parts.push_back({p + "o", vg});
      }
      if (s.latent) L.latent(*s.latent, l + s.latent->prefix, w);
      else w.out = L.columns(out_parts, W);
      auto norms = [&](const std::string& name, const std::string& scale, nf_norm& in, nf_norm& out) {
        const std::string columns = spec.layer_scale ? l + scale : "";
        if (spec.pre_norm) in = L.norm(l + name, spec.norm);
        if (!spec.pre_norm || spec.post_norm) out = L.norm(l + name + (spec.pre_norm ? "b" : ""), spec.norm, 1, columns);
      };
      norms("norm1", "ls1", w.norm1, w.out_norm1);
      if (s.hasFeedForward()) norms("norm2", "ls2", w.norm2, w.out_norm2);
      if (s.mlp) {
        w.up = L.matrix({{l + "mlp.up", s.mlp->ff}}, W);
        w.down = L.matrix({{l + "mlp.down", W}}, s.mlp->ff);
      }
      if (s.mixture) L.mixture(*s.mixture, l + "mlp.", w);
      if (spec.token_side > 0) {
        w.side_gate = L.matrix({{l + "side.gate", spec.token_side}}, W);
        w.side_proj = L.matrix({{l + "side.proj", W}}, spec.token_side);
        w.side_norm = L.norm(l + "side.norm", NF_NORM_RMS);
      }
    }
    for (size_t r = 0; r < runs.size(); ++r) {  // caches and states
      const int i = runs[r].layer;
      const LayerSpec& s = spec.layers[i];
      if (s.attention) {
        const nf_kv_layout kv = kvLayout(i);
        kv_data[r] = allocate((size_t)kv_pages * nf_kv_page_elements(&kv) * elementBytes());
        if (s.attention->conv_taps > 0)
          conv_state[r] = allocate((size_t)state_slots * (s.attention->conv_taps - 1) * weights.layers[i].attention.qkv.N * elementBytes());
      }
      if (s.latent) kv_data[r] = allocate((size_t)kv_pages * page_size * latentLayout(i).row_ld * elementBytes());
      if (s.recurrence) {
        state[r] = static_cast<float*>(allocate((size_t)state_slots * s.recurrence->heads *
                                                nf_recurrence_state_elements(s.recurrence->dim, s.recurrence->vdim) * sizeof(float)));
        if (s.recurrence->kind == NF_RECURRENCE_TOKEN_DECAY)
          shift_state[r] = static_cast<float*>(allocate((size_t)state_slots * ld * sizeof(float)));
      }
    }
  } catch (...) {
    for (void* p : owned_) (void)hipFree(p);
    owned_.clear();
    throw;
  }
}

StackModel::~StackModel() {
  for (void* p : owned_) (void)hipFree(p);
}
