#include "stackModel.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>
#include <cstring>
#include <stdexcept>

#include "helper.h"

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
  require(s.width > 0 && s.vocab > 0 && s.max_positions > 0 && !s.layers.empty(), "width, vocab, max_positions and layers must be positive");
  for (size_t i = 0; i < s.layers.size(); ++i) {
    const LayerSpec& l = s.layers[i];
    const std::string at = "layer " + std::to_string(i) + ": ";
    require(l.attention || l.recurrence, at + "no mixer");
    if (l.attention) {
      const auto& a = *l.attention;
      require(a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0, at + "query heads must be a multiple of the kv heads");
      require(a.dim > 0 && a.dim <= 256 && a.vdim > 0 && a.vdim <= 256, at + "attention head sizes must be in 1..256");
      require(a.rot.dims >= 0 && a.rot.dims <= a.dim && a.rot.dims % 2 == 0, at + "rotated dimensions");
      require(a.window >= 0 && a.keep_first >= 0, at + "window");
    }
    if (l.recurrence) {
      const auto& r = *l.recurrence;
      require(r.heads > 0 && r.dim > 0 && r.dim <= 256 && r.vdim > 0 && r.vdim <= 256, at + "recurrence head sizes must be in 1..256");
      require(r.rot.dims >= 0 && r.rot.dims <= r.dim && r.rot.dims % 2 == 0, at + "rotated dimensions");
      require(r.kind != NF_RECURRENCE_FIXED_DECAY || (int)r.decay.size() == r.heads, at + "one decay per head");
    }
    if (l.mlp) require(l.mlp->ff > 0, at + "feed-forward width");
  }
  return s;
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
  struct Part {
    std::string name;
    int rows;
  };
  void put_rows(const HostTensor& t, int rows, int cols, int row0, int col0, int K) {
    const size_t es = m.elementBytes();
    for (int r = 0; r < rows; ++r) {
      uint8_t* dst = staging.data() + ((size_t)(row0 + r) * K + col0) * es;
      if (m.dtype == NF_BF16 && t.type == HostTensor::BF16) {
        std::memcpy(dst, static_cast<const uint8_t*>(t.data) + (size_t)r * cols * 2, (size_t)cols * 2);
        continue;
      }
      for (int c = 0; c < cols; ++c) {
        const float f = element(t, (size_t)r * cols + c);
        if (m.dtype == NF_BF16) {
          const uint16_t b = float_to_bf16(f);
          std::memcpy(dst + 2 * c, &b, 2);
        } else {
          std::memcpy(dst + 4 * c, &f, 4);
        }
      }
    }
  }
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
    staging.assign((size_t)N * K * m.elementBytes(), 0);
    int at = 0;
    for (const auto& p : parts) {
      if (first_row) first_row->push_back(at);
      put_rows(get(p.name, {p.rows, cols}), p.rows, cols, at, 0, K);
      at += p.rows;
    }
    return finish(N, K);
  }
  // [rows][k_1 | k_2 | ...]: output projections of mixers side by side, applied to their concatenated heads
  DeviceMatrix columns(const std::vector<Part>& parts, int rows) {
    int cols = 0;
    for (const auto& p : parts) cols += p.rows;
    const int N = pad8(rows), K = pad8(cols);
    staging.assign((size_t)N * K * m.elementBytes(), 0);
    int at = 0;
    for (const auto& p : parts) {
      put_rows(get(p.name, {rows, p.rows}), rows, p.rows, 0, at, K);
      at += p.rows;
    }
    return finish(N, K);
  }
  float* upload(const std::vector<float>& v) {
    float* d = static_cast<float*>(m.allocate(v.size() * sizeof(float)));
    HIP_CHECK(hipMemcpy(d, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
    return d;
  }
  // vectors of `rows` x `cols`, each row padded to `ld`
  float* vectors(const std::vector<std::string>& names, std::vector<int64_t> shape, int cols, int ld) {
    std::vector<float> v((size_t)names.size() * ld, 0.f);
    for (size_t s = 0; s < names.size(); ++s) {
      const HostTensor& t = get(names[s], shape);
      for (int c = 0; c < cols; ++c) v[s * ld + c] = element(t, c);
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

// cos and sin of position * base^(-2i/dims), evaluated in double and kept in fp32: one table per distinct
// rotation, for every position a request can have.
nf_rotation StackModel::rotation(const RotationSpec& r) {
  nf_rotation out{nullptr, r.dims, r.interleaved ? 1 : 0};
  if (r.dims == 0) return out;
  float*& table = rotation_tables_[{r.dims, r.base}];
  if (!table) {
    const int half = r.dims / 2;
    std::vector<float> v((size_t)spec.max_positions * half * 2);
    for (int i = 0; i < half; ++i) {
      const double f = std::pow(r.base, -2.0 * i / r.dims);
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

nf_kv_layout StackModel::kvLayout(int layer) const {
  const AttentionSpec& a = *spec.layers[layer].attention;
  return nf_kv_layout{dtype, a.heads, a.kv_heads, a.dim, a.vdim, (a.dim + 31) / 32 * 32, (a.vdim + 15) / 16 * 16, page_size};
}

StackModel::StackModel(const StackModelSpec& spec_, const HostTensors& tensors, nf_dtype dtype_, int kv_pages_, int page_size_,
                       int state_slots_)
    : spec(spec_), dtype(dtype_), kv_pages(kv_pages_), page_size(page_size_), state_slots(state_slots_) {
  const int W = spec.width, ld = spec.ld();
  Loader L{*this, tensors, {}};
  try {
    weights.embed = L.matrix({{"embed", spec.vocab}}, W);
    if (spec.learned_positions) weights.pos = L.matrix({{"pos", spec.max_positions}}, W);
    weights.head = L.matrix({{"head", spec.vocab}}, W);
    weights.final_norm = L.vectors({"final.norm"}, {W}, W, ld);
    const int n = (int)spec.layers.size();
    weights.layers.resize(n);
    kv_data.assign(n, nullptr);
    state.assign(n, nullptr);
    shift_state.assign(n, nullptr);
    for (int i = 0; i < n; ++i) {
      const LayerSpec& s = spec.layers[i];
      LayerWeights& w = weights.layers[i];
      const std::string l = "l" + std::to_string(i) + ".";
      std::vector<Loader::Part> out_parts;
      if (s.attention) {
        const AttentionSpec& a = *s.attention;
        const std::string p = l + a.prefix;
        std::vector<int> at;
        w.attention.qkv = L.matrix({{p + "q", a.heads * a.dim}, {p + "k", a.kv_heads * a.dim}, {p + "v", a.kv_heads * a.vdim}}, W, &at);
        w.attention.q_col = at[0];
        w.attention.k_col = at[1];
        w.attention.v_col = at[2];
        if (a.qk_norm) {
          w.attention.q_norm = L.vectors({p + "q.norm"}, {a.dim}, a.dim, a.dim);
          w.attention.k_norm = L.vectors({p + "k.norm"}, {a.dim}, a.dim, a.dim);
        }
        if (a.sink) w.attention.sink = L.vectors({p + "sink"}, {a.heads}, a.heads, a.heads);
        w.attention.rot = rotation(a.rot);
        out_parts.push_back({p + "o", a.heads * a.vdim});
        const nf_kv_layout kv = kvLayout(i);
        kv_data[i] = allocate((size_t)kv_pages * nf_kv_page_elements(&kv) * elementBytes());
      }
      if (s.recurrence) {
        const RecurrenceSpec& r = *s.recurrence;
        const std::string p = l + r.prefix;
        const int qk = r.heads * r.dim, vg = r.heads * r.vdim;
        if (r.kind == NF_RECURRENCE_FIXED_DECAY) {
          std::vector<int> at;
          w.recurrence.qkvg = L.matrix({{p + "q", qk}, {p + "k", qk}, {p + "v", vg}, {p + "g", vg}}, W, &at);
          w.recurrence.q_col = at[0];
          w.recurrence.k_col = at[1];
          w.recurrence.v_col = at[2];
          w.recurrence.g_col = at[3];
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
          shift_state[i] = static_cast<float*>(allocate((size_t)state_slots * ld * sizeof(float)));
        }
        out_parts.push_back({p + "o", vg});
        state[i] = static_cast<float*>(
            allocate((size_t)state_slots * r.heads * nf_recurrence_state_elements(r.dim, r.vdim) * sizeof(float)));
      }
      w.out = L.columns(out_parts, W);
      w.norm1 = L.vectors({l + "norm1"}, {W}, W, ld);
      if (s.mlp) {
        w.up = L.matrix({{l + "mlp.up", s.mlp->ff}}, W);
        w.down = L.matrix({{l + "mlp.down", W}}, s.mlp->ff);
        w.norm2 = L.vectors({l + "norm2"}, {W}, W, ld);
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
