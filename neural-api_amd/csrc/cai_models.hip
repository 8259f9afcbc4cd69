// Model registry: a folder with config.json and model.safetensors is loaded by the builder registered under its
// "architecture"; a file is a GGUF container (cai_gguf.hip).  Host code only.
//
// A builder reads every size from the configuration or from a tensor's shape, checks the two against each other before anything
// is sized from them, stacks the projections that share an input into one matrix, and describes the layers to the layered
// decoder.
#include "cai_layered.hpp"
#include "cai_json.hpp"

#include <algorithm>
#include <fcntl.h>
#include <math.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <map>
#include <string>

namespace cai {

namespace {

// ------------------------------------------------------------------------------------------
// safetensors: an 8-byte little-endian header length, the JSON header (name -> dtype, shape, data_offsets), the data
// ------------------------------------------------------------------------------------------
struct StTensor { std::string dtype; std::vector<int64_t> shape; const uint8_t* data = nullptr; int64_t bytes = 0, elems = 1; };

struct SafeTensors {
  void* base = MAP_FAILED; size_t size = 0;
  std::map<std::string, StTensor> t;
  ~SafeTensors() { if (base != MAP_FAILED) munmap(base, size); }

  int open(const std::string& path)
  {
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return set_error(CAI_ERR_INVALID, "safetensors: cannot open %s", path.c_str());
    struct stat sb;
    if (fstat(fd, &sb) || sb.st_size < 8) { close(fd); return set_error(CAI_ERR_INVALID, "safetensors: %s is too short", path.c_str()); }
    size = (size_t)sb.st_size;
    base = mmap(nullptr, size, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (base == MAP_FAILED) return set_error(CAI_ERR_INVALID, "safetensors: cannot map %s", path.c_str());
    const uint8_t* p = (const uint8_t*)base;
    uint64_t hl = 0;
    memcpy(&hl, p, 8);
    if (hl > size - 8) return set_error(CAI_ERR_INVALID, "safetensors: header of %llu bytes in a file of %zu: %s", (unsigned long long)hl, size, path.c_str());
    Json j; std::string err;
    if (!JsonReader::parse((const char*)p + 8, (size_t)hl, j, err) || j.kind != Json::OBJ) return set_error(CAI_ERR_INVALID, "safetensors: %s: %s", err.c_str(), path.c_str());
    const uint64_t data0 = 8 + hl, room = size - data0;
    for (auto& kv : j.obj) {
      if (kv.first == "__metadata__") continue;
      const Json *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *of = kv.second.get("data_offsets");
      bool ok = dt && dt->kind == Json::STR && sh && sh->kind == Json::ARR && of && of->kind == Json::ARR && of->arr.size() == 2 && of->arr[0].is_int() && of->arr[1].is_int();
      StTensor x;
      if (ok) {
        x.dtype = dt->str;
        for (auto& d : sh->arr) {
          ok = ok && d.is_int() && d.num >= 0 && d.num < 2147483648.0 && x.elems < ((int64_t)1 << 40);
          if (ok) { x.shape.push_back((int64_t)d.num); x.elems *= (int64_t)d.num; }
        }
        const double a = of->arr[0].num, b = of->arr[1].num;
        const int64_t es = x.dtype == "BF16" || x.dtype == "F16" ? 2 : x.dtype == "F32" || x.dtype == "I32" ? 4 : 0;
        ok = ok && a >= 0 && b >= a && b <= (double)room && es > 0 && (int64_t)(b - a) == x.elems * es;
        if (ok) { x.data = p + data0 + (uint64_t)a; x.bytes = (int64_t)(b - a); }
      }
      if (!ok) return set_error(CAI_ERR_INVALID, "safetensors: tensor \"%s\" has a bad type, shape or range: %s", kv.first.c_str(), path.c_str());
      if (!t.emplace(kv.first, x).second) return set_error(CAI_ERR_INVALID, "safetensors: tensor \"%s\" is listed twice: %s", kv.first.c_str(), path.c_str());
    }
    return CAI_OK;
  }
};

// ------------------------------------------------------------------------------------------
// what every builder uses: checked access to configuration and tensors.  The first failure sticks in rc.
// ------------------------------------------------------------------------------------------
struct Builder {
  SafeTensors st;
  NetSpec s;
  int rc = CAI_OK;

  bool fail(const std::string& m) { if (!rc) rc = set_error(CAI_ERR_INVALID, "model: %s", m.c_str()); return false; }

  int integer(const Json* o, const char* key, const std::string& where, int lo = 1, int hi = 1 << 24)
  {
    const Json* v = o ? o->get(key) : nullptr;
    if (!v || !v->is_int() || v->num < lo || v->num > hi) { fail("\"" + where + key + "\" is missing or not an integer in " + std::to_string(lo) + ".." + std::to_string(hi)); return lo; }
    return (int)v->num;
  }
  float number(const Json* o, const char* key, const std::string& where)
  {
    const Json* v = o ? o->get(key) : nullptr;
    if (!v || v->kind != Json::NUM) { fail("\"" + where + key + "\" is missing or not a number"); return 0.0f; }
    return (float)v->num;
  }
  const StTensor* tensor(const std::string& name, std::vector<int64_t> shape)
  {
    auto it = st.t.find(name);
    if (it == st.t.end()) { fail("missing tensor \"" + name + "\""); return nullptr; }
    bool ok = it->second.shape.size() == shape.size();
    for (size_t i = 0; ok && i < shape.size(); i++) ok = shape[i] < 0 ? it->second.shape[i] > 0 : it->second.shape[i] == shape[i];
    if (!ok) {
      std::string a, b;
      for (int64_t v : it->second.shape) a += (a.empty() ? "" : "x") + std::to_string(v);
      for (int64_t v : shape) b += (b.empty() ? "" : "x") + (v < 0 ? std::string("?") : std::to_string(v));
      fail("tensor \"" + name + "\" is [" + a + "], expected [" + b + "]");
      return nullptr;
    }
    return &it->second;
  }
  bool floats(const std::string& name, std::vector<int64_t> shape, std::vector<float>& out)
  {
    const StTensor* t = tensor(name, shape);
    if (!t) return false;
    out.resize((size_t)t->elems);
    if (t->dtype == "F32") memcpy(out.data(), t->data, (size_t)t->bytes);
    else if (t->dtype == "BF16") for (int64_t i = 0; i < t->elems; i++) { uint16_t b; memcpy(&b, t->data + 2 * i, 2); const uint32_t u = (uint32_t)b << 16; memcpy(&out[i], &u, 4); }
    else return fail("tensor \"" + name + "\" has type " + t->dtype + ", expected BF16 or F32");
    return true;
  }
  template <typename T> T* upload(const std::vector<T>& v)
  {
    if (rc) return nullptr;
    void* p = nullptr;
    hipError_t e = hipMalloc(&p, v.size() * sizeof(T));
    if (e == hipSuccess) { s.vectors.push_back(p); e = hipMemcpy(p, v.data(), v.size() * sizeof(T), hipMemcpyHostToDevice); }
    if (e != hipSuccess) { rc = hip_fail(e, "model vector upload", __FILE__, __LINE__); return nullptr; }
    return (T*)p;
  }
  float* vec(const std::string& name, std::vector<int64_t> shape)
  {
    std::vector<float> v;
    return floats(name, shape, v) ? upload(v) : nullptr;
  }
  // rows of several matrices of one width, one after the other; order (may be null) gives the source row of each resident row,
  // -1 a row of zeros
  cai_qw_s* stack(const std::vector<std::pair<std::string, int64_t>>& parts, int64_t cols, const std::vector<int>* order = nullptr)
  {
    if (rc) return nullptr;
    int64_t rows = 0;
    std::vector<const uint8_t*> src;
    for (auto& p : parts) {
      const StTensor* t = tensor(p.first, {p.second, cols});
      if (!t) return nullptr;
      if (t->dtype != "BF16") { fail("tensor \"" + p.first + "\" has type " + t->dtype + ", expected BF16"); return nullptr; }
      for (int64_t r = 0; r < p.second; r++) src.push_back(t->data + r * cols * 2);
      rows += p.second;
    }
    if (order) {
      std::vector<const uint8_t*> re(order->size());
      for (size_t i = 0; i < order->size(); i++) re[i] = (*order)[i] < 0 ? nullptr : src[(size_t)(*order)[i]];
      src.swap(re); rows = (int64_t)src.size();
    }
    std::vector<uint8_t> buf((size_t)(rows * cols * 2));
    for (int64_t r = 0; r < rows; r++) { if (src[r]) memcpy(buf.data() + r * cols * 2, src[r], (size_t)cols * 2); else memset(buf.data() + r * cols * 2, 0, (size_t)cols * 2); }
    cai_qw_t w = nullptr;
    if ((rc = cai_qw_create(CAI_BF16, rows, cols, buf.data(), nullptr, &w))) return nullptr;
    s.weights.push_back(w);
    return w;
  }
  // mult: a constant the norm's result is multiplied by, carried in its weight and bias
  Dyt dyt_norm(const std::string& name, int width, float mult = 1.0f)
  {
    Dyt d;
    std::vector<float> a, w, b;
    if (!floats(name + ".alpha", {}, a) || !floats(name, {width}, w) || !floats(name + ".b", {width}, b)) return d;
    for (float& v : w) v *= mult;
    for (float& v : b) v *= mult;
    d.alpha = a[0]; d.w = upload(w); d.b = upload(b);
    return d;
  }
  // gate and up matrices of one or several feed-forwards (names end before "gate"), rows interleaved in blocks of 16, one after the other
  cai_qw_s* gated(const std::vector<std::string>& pre, int ff, int width)
  {
    std::vector<std::pair<std::string, int64_t>> parts;
    std::vector<int> order((size_t)pad_to(ff, 16) * 2 * pre.size(), -1);
    for (size_t e = 0; e < pre.size(); e++) {
      parts.push_back({pre[e] + "gate", ff}); parts.push_back({pre[e] + "up", ff});
      const size_t base = e * (size_t)pad_to(ff, 16) * 2;
      for (int j = 0; j < ff; j++) { order[base + glu_row(j, 0)] = (int)(2 * e) * ff + j; order[base + glu_row(j, 1)] = (int)(2 * e + 1) * ff + j; }
    }
    return stack(parts, width, &order);
  }
  // matrices of equal shape one after the other, each padded to whole blocks of 16 rows with zeros
  cai_qw_s* padded_bank(const std::vector<std::string>& names, int rows, int width)
  {
    std::vector<std::pair<std::string, int64_t>> parts;
    std::vector<int> order((size_t)pad_to(rows, 16) * names.size(), -1);
    for (size_t e = 0; e < names.size(); e++) {
      parts.push_back({names[e], rows});
      for (int j = 0; j < rows; j++) order[e * pad_to(rows, 16) + j] = (int)e * rows + j;
    }
    return stack(parts, width, &order);
  }
  // the experts' matrices, one after the other
  void banks(const std::string& pre, int n, int ff, int width, NetExperts& x)
  {
    std::vector<std::string> names; std::vector<std::pair<std::string, int64_t>> down;
    for (int i = 0; i < n; i++) { names.push_back(pre + "e" + std::to_string(i) + "."); down.push_back({names.back() + "down", width}); }
    if (x.gated) x.gateup = gated(names, ff, width);
    else { for (auto& s : names) s += "up"; x.gateup = padded_bank(names, ff, width); }
    x.down = stack(down, ff);
  }
  // a rotation's rates: turns a position of each pair of the first `dims` dimensions, base^(-2i/dims) radians divided by `linear`.  yarn:
  // pairs that make less than `slow` turns over `original` positions are divided by `factor`, those that make more than `fast` are not,
  // with a ramp in between (slow and fast turned into pair numbers, rounded outwards)
  struct Yarn { double factor, original, fast, slow; };
  const double* rates(int dims, double base, double linear, const Yarn* y)
  {
    std::vector<double> turns((size_t)dims / 2);
    double lo = 0.0, hi = 0.0;
    if (y) {
      auto pair = [&](double t) { return dims * log(y->original / (2.0 * M_PI * t)) / (2.0 * log(base)); };
      lo = std::max(floor(pair(y->fast)), 0.0); hi = std::min(ceil(pair(y->slow)), dims - 1.0);
    }
    for (int i = 0; i < dims / 2; i++) {
      const double f = pow(base, -2.0 * i / dims) / (2.0 * M_PI) / linear;
      const double ramp = y ? std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0) : 0.0;
      turns[i] = y ? f / y->factor * ramp + f * (1.0 - ramp) : f;
    }
    return dims ? upload(turns) : nullptr;
  }
  // sizes every layered design has, and its list of layers; may_loop: a stretch of layers may run several times; tied: the embedding
  // table is the matrix of the logits too
  const Json* layer_list(const Json& cfg, bool may_loop, bool tied = false)
  {
    s.width = integer(&cfg, "width", ""); s.vocab = integer(&cfg, "vocab", "", 1, 1 << 28);
    s.eps = number(cfg.get("norm"), "eps", "norm.");
    const Json* layers = cfg.get("layers");
    if (!layers || layers->kind != Json::ARR || layers->arr.empty()) { fail("\"layers\" is missing or empty"); return nullptr; }
    const int L = (int)layers->arr.size();
    const Json* loop = may_loop ? cfg.get("loop") : nullptr;
    if (loop && loop->kind != Json::NUL) {
      s.loop_start = integer(loop, "start", "loop.", 0, L); s.loop_stop = integer(loop, "stop", "loop.", 0, L); s.loop_times = integer(loop, "times", "loop.", 1, 4096);
      if (!rc && s.loop_stop < s.loop_start) fail("loop.stop lies before loop.start");
    }
    if (rc) return nullptr;
    s.embed = stack({{"embed", s.vocab}}, s.width);
    s.head = tied ? s.embed : stack({{"head", s.vocab}}, s.width);
    return rc ? nullptr : layers;
  }
  std::string word(const Json* o, const char* key) { const Json* v = o ? o->get(key) : nullptr; return v && v->kind == Json::STR ? v->str : std::string(); }
};

// ------------------------------------------------------------------------------------------
// Samanex: gated-delta-rule layers and layers of a windowed attention beside a delta rule with a decay per key channel; Dynamic
// Tanh before and after each sublayer; a stretch of layers repeated with the embedding output added in front of each repeat.
// ------------------------------------------------------------------------------------------
void delta_block(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, bool channel, NetDelta& D,
                 std::vector<std::pair<std::string, int64_t>>& parts, int& at)
{
  DeltaDims& d = D.d;
  d.heads = b.integer(c, "heads", where, 1, 65535); d.kv_heads = b.integer(c, "kv_heads", where, 1, 65535);
  d.dim = b.integer(c, "dim", where, 1, 256); d.vdim = b.integer(c, "vdim", where, 1, 256); d.taps = b.integer(c, "conv", where, 1, 4096);
  d.eps = b.s.eps; d.channel_decay = channel; d.sigmoid_gate = channel;
  if (b.rc) return;
  if (d.heads % d.kv_heads) { b.fail(where + "heads is not a multiple of " + where + "kv_heads"); return; }
  const int kw = d.kv_heads * d.dim, vw = d.heads * d.vdim;
  auto take = [&](const char* n, int rows) { const int o = at; parts.push_back({pre + n, rows}); at += rows; return o; };
  D.oq = take("q", kw); D.ok = take("k", kw); D.ov = take("v", vw); D.ob = take("b", d.heads);
  if (channel) {
    const StTensor *a1 = b.tensor(pre + "a1", {-1, width}), *g1 = b.tensor(pre + "g1", {-1, width});
    if (!a1 || !g1) return;
    d.rank_a = (int)a1->shape[0]; d.rank_g = (int)g1->shape[0];
    if (d.rank_a > 512 || d.rank_g > 512) { b.fail(where + "low-rank projections of more than 512 rows"); return; }
    D.oa = take("a1", d.rank_a); D.og = take("g1", d.rank_g);
    D.w.a2 = b.stack({{pre + "a2", (int64_t)d.heads * d.dim}}, d.rank_a);
    D.w.g2 = b.stack({{pre + "g2", vw}}, d.rank_g);
    D.w.dt_bias = b.vec(pre + "dt_bias", {(int64_t)d.heads * d.dim});
  } else {
    D.oa = take("a", d.heads); D.og = take("g", vw);
    D.w.dt_bias = b.vec(pre + "dt_bias", {d.heads});
  }
  D.w.cq = b.vec(pre + "q.conv", {kw, d.taps}); D.w.ck = b.vec(pre + "k.conv", {kw, d.taps}); D.w.cv = b.vec(pre + "v.conv", {vw, d.taps});
  std::vector<float> al;
  if (!b.floats(pre + "A_log", {d.heads}, al)) return;
  for (float& v : al) v = -expf(v);
  D.w.rate = b.upload(al);
  D.w.norm = b.vec(pre + "norm", {d.vdim});
  D.out = b.stack({{pre + "o", width}}, vw);
}

void attn_block(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetAttn& A,
                std::vector<std::pair<std::string, int64_t>>& parts, int& at)
{
  AttnDims& d = A.d;
  d.heads = b.integer(c, "heads", where, 1, 65535); d.kv_heads = b.integer(c, "kv_heads", where, 1, 65535);
  d.dim = b.integer(c, "dim", where, 1, 256); d.vdim = b.integer(c, "vdim", where, 1, 256);
  d.window = b.integer(c ? c->get("mask") : nullptr, "size", where + "mask.", 1, 1 << 30);
  d.scale = b.number(c, "scale", where); d.eps = b.s.eps;
  d.dim_p = pad_to(d.dim, 8); d.vdim_p = pad_to(d.vdim, 8);
  if (b.rc) return;
  if (d.heads % d.kv_heads) { b.fail(where + "heads is not a multiple of " + where + "kv_heads"); return; }
  auto take = [&](const char* n, int rows) { const int o = at; parts.push_back({pre + n, rows}); at += rows; return o; };
  A.oq = take("q", d.heads * d.dim); A.ok = take("k", d.kv_heads * d.dim); A.ov = take("v", d.kv_heads * d.vdim);
  A.qn = b.vec(pre + "q.norm", {d.dim}); A.kn = b.vec(pre + "k.norm", {d.dim}); A.og = -1;
  A.out = b.stack({{pre + "o", width}}, (int64_t)d.heads * d.vdim);
}

void build_samanex(Builder& b, const Json& cfg)
{
  NetSpec& s = b.s;
  const Json* layers = b.layer_list(cfg, true);
  if (!layers) return;
  s.final_norm = b.dyt_norm("final.norm", s.width);
  const int L = (int)layers->arr.size(), w = s.width;
  for (int l = 0; l < L && !b.rc; l++) {
    const Json& c = layers->arr[l];
    const std::string p = "l" + std::to_string(l) + ".", where = "layers[" + std::to_string(l) + "].";
    const Json *type = c.get("type"), *mix = c.get("mixer"), *mlp = c.get("mlp");
    NetLayer y;
    std::vector<std::pair<std::string, int64_t>> parts; int at = 0;
    if (type && type->kind == Json::STR && type->str == "delta") {
      y.kind = MIX_DELTA;
      delta_block(b, mix, where + "mixer.", p + "mix.", w, false, y.delta, parts, at);
    } else if (type && type->kind == Json::STR && type->str == "parallel") {
      y.kind = MIX_PARALLEL;
      attn_block(b, mix ? mix->get("left") : nullptr, where + "mixer.left.", p + "mix.left.", w, y.attn, parts, at);
      if (!b.rc) delta_block(b, mix ? mix->get("right") : nullptr, where + "mixer.right.", p + "mix.right.", w, true, y.delta, parts, at);
      y.gain_left = b.vec(p + "mix.left.out", {w}); y.gain_right = b.vec(p + "mix.right.out", {w});
    } else b.fail("\"" + where + "type\" is not one of delta, parallel");
    if (b.rc) return;
    y.in = b.stack(parts, w);
    y.norm1 = b.dyt_norm(p + "norm1", w); y.norm1b = b.dyt_norm(p + "norm1b", w);
    if (mlp && mlp->kind == Json::OBJ) {
      const Json* kind = mlp->get("kind");
      if (!kind || kind->kind != Json::STR || kind->str != "dense") { b.fail("\"" + where + "mlp.kind\" is not dense"); return; }
      y.ff = b.integer(mlp, "ff", where + "mlp.");
      if (b.rc) return;
      y.norm2 = b.dyt_norm(p + "norm2", w); y.norm2b = b.dyt_norm(p + "norm2b", w);
      y.gateup = b.gated({p + "mlp."}, y.ff, w);
      y.down = b.stack({{p + "mlp.down", w}}, y.ff);
      y.glu = GLU_RELU;
    } else if (mlp && mlp->kind != Json::NUL) b.fail("\"" + where + "mlp\" is neither an object nor null");
    s.layers.push_back(y);
  }
}

// ------------------------------------------------------------------------------------------
// Kiruvik: rotary attention in fixed blocks of positions with an output gate, and Mamba-2 layers; dense or mixture-of-experts
// feed-forwards; Dynamic Tanh before and after each sublayer, the latter times one constant; a stretch of layers run several times,
// a matrix over the stream and the embedding output in front of every pass.
// ------------------------------------------------------------------------------------------
void block_attention(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetLayer& y)
{
  NetAttn& A = y.attn; AttnDims& d = A.d;
  d.heads = b.integer(c, "heads", where, 1, 65535); d.kv_heads = b.integer(c, "kv_heads", where, 1, 65535);
  d.dim = b.integer(c, "dim", where, 1, 256); d.vdim = b.integer(c, "vdim", where, 1, 256);
  const Json *mask = c ? c->get("mask") : nullptr, *rot = c ? c->get("rot") : nullptr;
  d.window = b.integer(mask, "size", where + "mask.", 1, 1 << 30); d.chunked = 1;
  d.rot = b.integer(rot, "dims", where + "rot.", 0, d.dim);
  const float base = b.number(rot, "base", where + "rot.");
  d.scale = b.number(c, "scale", where); d.eps = b.s.eps;
  d.dim_p = pad_to(d.dim, 8); d.vdim_p = pad_to(d.vdim, 8);
  if (b.rc) return;
  if (d.heads % d.kv_heads) { b.fail(where + "heads is not a multiple of " + where + "kv_heads"); return; }
  if (d.rot % 2 || !(base > 0.0f)) { b.fail(where + "rot needs an even number of dims and a base above zero"); return; }
  d.turns = b.rates(d.rot, rot->get("base")->num, 1.0, nullptr);
  const int qw = d.heads * d.dim, kw = d.kv_heads * d.dim, vw = d.kv_heads * d.vdim, ow = d.heads * d.vdim;
  A.oq = 0; A.ok = qw; A.ov = qw + kw; A.og = qw + kw + vw;
  y.in = b.stack({{pre + "q", qw}, {pre + "k", kw}, {pre + "v", vw}, {pre + "g", ow}}, width);
  std::vector<float> bias, part;
  for (auto& n : {std::make_pair("q.b", qw), std::make_pair("k.b", kw), std::make_pair("v.b", vw)}) {
    if (!b.floats(pre + n.first, {n.second}, part)) return;
    bias.insert(bias.end(), part.begin(), part.end());
  }
  bias.resize((size_t)A.og + ow, 0.0f);                  // (the gate has none)
  y.in_b = b.upload(bias);
  A.out = b.stack({{pre + "o", width}}, ow);
  A.out_b = b.vec(pre + "o.b", {width});
}

void ssd_block(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetLayer& y)
{
  NetSsd& M = y.ssd; SsdDims& d = M.d;
  d.heads = b.integer(c, "heads", where, 1, 65535); d.vdim = b.integer(c, "vdim", where, 1, 256); d.state = b.integer(c, "state", where, 1, 256);
  d.groups = b.integer(c, "groups", where, 1, 65535); d.taps = b.integer(c, "conv", where, 1, 4096); d.norm_groups = b.integer(c, "norm_groups", where, 1, 65535);
  d.eps = b.s.eps;
  if (b.rc) return;
  if (d.heads % d.groups) { b.fail(where + "heads is not a multiple of " + where + "groups"); return; }
  if (d.inner() % d.norm_groups) { b.fail("heads times vdim is not a multiple of " + where + "norm_groups"); return; }
  M.oz = 0; M.ox = d.inner(); M.odt = M.ox + d.channels();
  y.in = b.stack({{pre + "in", (int64_t)M.odt + d.heads}}, width);
  M.w.conv = b.vec(pre + "conv", {d.channels(), d.taps}); M.w.conv_b = b.vec(pre + "conv.b", {d.channels()});
  M.w.dt_bias = b.vec(pre + "dt_bias", {d.heads}); M.w.D = b.vec(pre + "D", {d.heads}); M.w.norm = b.vec(pre + "norm", {d.inner()});
  std::vector<float> al;
  if (!b.floats(pre + "A_log", {d.heads}, al)) return;
  for (float& v : al) v = -expf(v);
  M.w.rate = b.upload(al);
  M.out = b.stack({{pre + "o", width}}, d.inner());
}

void experts_block(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetExperts& x)
{
  const Json *r = c->get("router"), *e = c->get("expert"), *sh = c->get("shared");
  const int n = b.integer(r, "experts", where + "router.", 1, EXPERTS_MAX);
  x.top = b.integer(r, "top", where + "router.", 1, std::min(n, EXPERTS_TOP)); x.scale = b.number(r, "scale", where + "router.");
  x.ff = b.integer(e, "ff", where + "expert."); x.limit = b.number(e, "limit", where + "expert.");
  if (b.rc) return;
  x.glu = x.glu_shared = GLU_CLAMPED;
  x.router = b.stack({{pre + "router", n}}, width);
  x.correction = b.vec(pre + "correction", {n});
  b.banks(pre, n, x.ff, width, x);
  if (sh && sh->kind != Json::NUL) {
    x.ff_shared = b.integer(sh, "ff", where + "shared."); x.limit_shared = b.number(sh, "limit", where + "shared.");
    if (b.rc) return;
    x.s_gateup = b.gated({pre + "shared."}, x.ff_shared, width);
    x.s_down = b.stack({{pre + "shared.down", width}}, x.ff_shared);
  }
  x.n = n;
}

void build_kiruvik(Builder& b, const Json& cfg)
{
  NetSpec& s = b.s;
  const Json* layers = b.layer_list(cfg, true);
  const float mult = b.number(&cfg, "residual_mult", "");
  if (!layers || b.rc) return;
  s.final_norm = b.dyt_norm("final.norm", s.width);
  const int L = (int)layers->arr.size(), w = s.width;
  if (s.loop_stop > s.loop_start) s.loop_in = b.stack({{"loop.in", w}}, 2 * w);
  for (int l = 0; l < L && !b.rc; l++) {
    const Json& c = layers->arr[l];
    const std::string p = "l" + std::to_string(l) + ".", where = "layers[" + std::to_string(l) + "].", type = b.word(&c, "type");
    const Json *mix = c.get("mixer"), *mlp = c.get("mlp");
    NetLayer y;
    if (type == "attention") { y.kind = MIX_ATTN; block_attention(b, mix, where + "mixer.", p + "mix.", w, y); }
    else if (type == "mamba2") { y.kind = MIX_SSD; ssd_block(b, mix, where + "mixer.", p + "mix.", w, y); }
    else b.fail("\"" + where + "type\" is not one of attention, mamba2");
    if (b.rc) return;
    y.norm1 = b.dyt_norm(p + "norm1", w); y.norm1b = b.dyt_norm(p + "norm1b", w, mult);
    if (mlp && mlp->kind == Json::OBJ) {
      const std::string kind = b.word(mlp, "kind");
      if (kind == "dense") {
        y.ff = b.integer(mlp, "ff", where + "mlp.");
        if (b.rc) return;
        y.gateup = b.gated({p + "mlp."}, y.ff, w);
        y.down = b.stack({{p + "mlp.down", w}}, y.ff);
        y.glu = GLU_GELU_TANH;
      } else if (kind == "moe") experts_block(b, mlp, where + "mlp.", p + "mlp.", w, y.experts);
      else b.fail("\"" + where + "mlp.kind\" is not one of dense, moe");
      if (b.rc) return;
      y.norm2 = b.dyt_norm(p + "norm2", w); y.norm2b = b.dyt_norm(p + "norm2b", w, mult);
    } else if (mlp && mlp->kind != Json::NUL) b.fail("\"" + where + "mlp\" is neither an object nor null");
    s.layers.push_back(y);
  }
}

// ------------------------------------------------------------------------------------------
// Gamanex: attention with sigmoid weights over every earlier key, the feed-forward (squared ReLU, or a mixture of experts) beside it on
// the same stream, both gated by a matrix over their own input.  A layer may attend over an earlier layer's keys and values.
// ------------------------------------------------------------------------------------------
void sigmoid_attention(Builder& b, const Json* c, const std::string& where, const std::string& p, int width, int layer, NetLayer& y)
{
  NetAttn& A = y.attn; AttnDims& d = A.d;
  const std::string pre = p + "mix.";
  d.heads = b.integer(c, "heads", where, 1, 65535); d.kv_heads = b.integer(c, "kv_heads", where, 1, 65535);
  d.dim = b.integer(c, "dim", where, 1, 256); d.vdim = b.integer(c, "vdim", where, 1, 256);
  d.scale = b.number(c, "scale", where); d.eps = b.s.eps; d.window = ATTN_EVERY_KEY;
  const Json *temp = c ? c->get("q_temp") : nullptr, *from = c ? c->get("kv_from") : nullptr;
  if (temp && temp->kind != Json::NUL) { d.temp = b.number(temp, "coef", where + "q_temp."); d.temp_every = b.integer(temp, "every", where + "q_temp.", 1, 1 << 30); }
  d.dim_p = pad_to(d.dim, 8); d.vdim_p = pad_to(d.vdim, 8); d.whole_norm = 1; d.sigmoid = 1;
  if (b.rc) return;
  if (d.heads % d.kv_heads) { b.fail(where + "heads is not a multiple of " + where + "kv_heads"); return; }
  if (from && from->kind != Json::NUL) {
    y.kv_from = b.integer(c, "kv_from", where, 0, 1 << 24);
    if (b.rc) return;
    if (y.kv_from >= layer || b.s.layers[y.kv_from].kv_from >= 0) { b.fail(where + "kv_from is not an earlier layer with keys and values of its own"); return; }
    const AttnDims& o = b.s.layers[y.kv_from].attn.d;
    if (o.heads != d.heads || o.kv_heads != d.kv_heads || o.dim != d.dim || o.vdim != d.vdim) { b.fail(where + "kv_from is a layer of other head counts or sizes"); return; }
  }
  const bool own = y.kv_from < 0;
  const int qw = d.heads * d.dim, kw = d.kv_heads * d.dim, vw = d.kv_heads * d.vdim;
  std::vector<std::pair<std::string, int64_t>> parts = {{p + "rg1", width}, {pre + "q", qw}};
  A.oq = width; A.ok = A.ov = A.og = -1;
  if (own) { A.ok = width + qw; A.ov = A.ok + kw; parts.push_back({pre + "k", kw}); parts.push_back({pre + "v", vw}); }
  y.in = b.stack(parts, width);
  std::vector<float> bias;
  if (!b.floats(p + "rg1.b", {width}, bias)) return;
  bias.resize((size_t)width + qw + (own ? kw + vw : 0), 0.0f);   // (the projections have none)
  y.in_b = b.upload(bias);
  A.qn = b.vec(pre + "q.norm", {qw});
  if (own) A.kn = b.vec(pre + "k.norm", {kw});
  d.r1 = b.vec(pre + "r1", {d.heads}); d.r2 = b.vec(pre + "r2", {d.heads}); d.bias = b.vec(pre + "pb", {d.heads});
  A.out = b.stack({{pre + "o", width}}, (int64_t)d.heads * d.vdim);
}

void build_gamanex(Builder& b, const Json& cfg)
{
  NetSpec& s = b.s;
  const Json* layers = b.layer_list(cfg, false);
  if (!layers) return;
  s.logit_scale = b.number(&cfg, "logit_scale", "");
  const int L = (int)layers->arr.size(), w = s.width;
  s.rms_final = b.vec("final.norm", {w});
  for (int l = 0; l < L && !b.rc; l++) {
    const Json& c = layers->arr[l];
    const std::string p = "l" + std::to_string(l) + ".", where = "layers[" + std::to_string(l) + "].";
    const Json* mlp = c.get("mlp");
    NetLayer y;
    y.beside = true; y.kind = MIX_ATTN;
    if (b.word(&c, "type") != "attention") { b.fail("\"" + where + "type\" is not attention"); return; }
    sigmoid_attention(b, c.get("mixer"), where + "mixer.", p, w, l, y);
    y.rms1 = b.vec(p + "norm1", {w}); y.scale1 = b.vec(p + "ls1", {w});
    if (b.rc) return;
    if (mlp && mlp->kind == Json::OBJ) {
      const std::string kind = b.word(mlp, "kind"), m = p + "mlp.", at = where + "mlp.";
      std::vector<float> bias, part;
      if (!b.floats(p + "rg2.b", {w}, bias)) return;
      if (kind == "dense") {
        y.ff = b.integer(mlp, "ff", at);
        if (b.rc) return;
        y.in2 = b.stack({{p + "rg2", w}, {m + "up", y.ff}}, w);
        y.down = b.stack({{m + "down", w}}, y.ff);
        bias.resize((size_t)w + y.ff, 0.0f);
      } else if (kind == "moe") {
        NetExperts& x = y.experts;
        const Json *r = mlp->get("router"), *e = mlp->get("expert");
        const int n = b.integer(r, "experts", at + "router.", 1, EXPERTS_MAX);
        x.top = b.integer(r, "top", at + "router.", 1, std::min(n, EXPERTS_TOP)); x.ff = b.integer(e, "ff", at + "expert.");
        if (b.rc) return;
        x.route = ROUTE_AMONG; x.glu = GLU_SILU;
        y.in2 = b.stack({{p + "rg2", w}, {m + "router", n}}, w);
        if (!b.floats(m + "router.b", {n}, part)) return;
        bias.insert(bias.end(), part.begin(), part.end());
        b.banks(m, n, x.ff, w, x);
        x.n = n;
      } else { b.fail("\"" + at + "kind\" is not one of dense, moe"); return; }
      y.in2_b = b.upload(bias);
      y.rms2 = b.vec(p + "norm2", {w}); y.scale2 = b.vec(p + "ls2", {w});
    } else if (mlp && mlp->kind != Json::NUL) b.fail("\"" + where + "mlp\" is neither an object nor null");
    s.layers.push_back(y);
  }
}

// ------------------------------------------------------------------------------------------
// Zenorax: latent attention, attention whose values are its keys, and linear attention with forget gates; mixtures of experts without
// gates, routed by sigmoids within groups; every sublayer between RMS norms, a convolution over time in front of every mixer, and a
// weighted sum of the results of all layers so far behind every layer.
// ------------------------------------------------------------------------------------------
bool rotation(Builder& b, const Json* rot, const std::string& where, int most, int& dims, double& base)
{
  dims = b.integer(rot, "dims", where, 0, most);
  b.number(rot, "base", where);
  if (b.rc) return false;
  base = rot->get("base")->num;
  if (dims % 2 || !(base > 0.0) || base == 1.0) return b.fail(where + "dims is odd, or " + where + "base no base of powers");
  return true;
}
const Json* present(const Json* o, const char* key) { const Json* v = o ? o->get(key) : nullptr; return v && v->kind != Json::NUL ? v : nullptr; }

void latent_attention(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetLayer& y)
{
  NetLatent& L = y.latent; LatentDims& d = L.d;
  d.heads = b.integer(c, "heads", where, 1, 65534); d.dim = b.integer(c, "dim", where, 1, 256); d.rot_dim = b.integer(c, "rot_dim", where, 0, 256);
  d.vdim = b.integer(c, "vdim", where, 1, 1024); d.q_rank = b.integer(c, "q_rank", where); d.kv_rank = b.integer(c, "kv_rank", where, 1, 768);
  d.scale = b.number(c, "scale", where); d.eps = b.s.eps; d.amp = 1.0f;
  const Json* rot = c ? c->get("rot") : nullptr;
  double base = 0.0;
  if (b.rc || !rotation(b, rot, where + "rot.", d.rot_dim, d.rot, base)) return;
  if (const Json* sc = present(rot, "scaling")) {
    for (const char* k : {"factor", "original", "fast", "slow"}) b.number(sc, k, where + "rot.scaling.");
    if (b.rc) return;
    const Builder::Yarn yarn{sc->get("factor")->num, sc->get("original")->num, sc->get("fast")->num, sc->get("slow")->num};
    if (!(yarn.factor > 0.0 && yarn.original > 0.0 && yarn.fast > 0.0 && yarn.slow > 0.0)) { b.fail(where + "rot.scaling has a number that is not above zero"); return; }
    d.turns = b.rates(d.rot, base, 1.0, &yarn);
    d.amp = (float)(0.1 * log(yarn.factor) + 1.0);
  } else d.turns = b.rates(d.rot, base, 1.0, nullptr);
  const int ow = d.heads * d.vdim;
  L.oq = 0; L.okv = d.q_rank; L.og = L.okv + d.kv_rank + d.rot_dim;
  y.in = b.stack({{pre + "dq", d.q_rank}, {pre + "dkv", d.kv_rank + d.rot_dim}, {pre + "g", ow}}, width);
  L.qn = b.vec(pre + "dq.norm", {d.q_rank}); L.kvn = b.vec(pre + "dkv.norm", {d.kv_rank});
  L.uq = b.stack({{pre + "uq", (int64_t)d.heads * (d.dim + d.rot_dim)}}, d.q_rank);
  // per head the rows of uk, then those of uv, each padded to eight
  std::vector<int> order((size_t)d.heads * d.head_e(), -1);
  for (int h = 0; h < d.heads; h++) {
    for (int i = 0; i < d.dim; i++) order[(size_t)h * d.head_e() + i] = h * d.dim + i;
    for (int i = 0; i < d.vdim; i++) order[(size_t)h * d.head_e() + d.dim_e() + i] = d.heads * d.dim + h * d.vdim + i;
  }
  L.up = b.stack({{pre + "uk", (int64_t)d.heads * d.dim}, {pre + "uv", ow}}, d.kv_rank, &order);
  L.out = b.stack({{pre + "o", width}}, ow);
  AttnDims& a = y.attn.d;                  // (the pages: one row of latent and turned part a token)
  a.heads = d.heads; a.kv_heads = 1; a.dim = a.dim_p = d.lat_p(); a.window = ATTN_EVERY_KEY;
}

// Queries and keys are normed behind the rotation; it leaves a head's length as it is, so the norm in front of it, with a gain of ones, is
// the same.
void key_value_attention(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetLayer& y)
{
  NetAttn& A = y.attn; AttnDims& d = A.d;
  d.heads = b.integer(c, "heads", where, 1, 65535); d.kv_heads = b.integer(c, "kv_heads", where, 1, 65535);
  d.dim = b.integer(c, "dim", where, 1, 256); d.vdim = b.integer(c, "vdim", where, 1, 256);
  d.scale = b.number(c, "scale", where); d.eps = b.s.eps; d.window = ATTN_EVERY_KEY;
  d.dim_p = pad_to(d.dim, 8); d.vdim_p = pad_to(d.vdim, 8);
  const Json* rot = c ? c->get("rot") : nullptr;
  double base = 0.0, linear = 1.0;
  if (b.rc || !rotation(b, rot, where + "rot.", d.dim, d.rot, base)) return;
  if (const Json* sc = present(rot, "scaling")) {
    b.number(sc, "factor", where + "rot.scaling.");
    if (b.rc) return;
    linear = sc->get("factor")->num;
    if (!(linear > 0.0)) { b.fail(where + "rot.scaling.factor is not above zero"); return; }
  }
  if (d.heads % d.kv_heads) { b.fail(where + "heads is not a multiple of " + where + "kv_heads"); return; }
  if (d.vdim != d.dim) { b.fail(where + "vdim is not " + where + "dim, but the values are the keys"); return; }
  d.turns = b.rates(d.rot, base, linear, nullptr);
  const int qw = d.heads * d.dim;
  A.oq = 0; A.ok = A.ov = qw; A.og = -1;
  y.in = b.stack({{pre + "q", qw}, {pre + "k", (int64_t)d.kv_heads * d.dim}}, width);
  A.qn = A.kn = b.upload(std::vector<float>(d.dim, 1.0f));
  d.sink = b.vec(pre + "sink", {d.heads});
  A.out = b.stack({{pre + "o", width}}, qw);
}

void forget_gate_attention(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetLayer& y)
{
  NetGla& G = y.gla; GlaDims& d = G.d;
  d.heads = b.integer(c, "heads", where, 1, 65535); d.dim = b.integer(c, "dim", where, 1, 256); d.vdim = b.integer(c, "vdim", where, 1, 256);
  d.eps = b.s.eps;
  if (b.rc) return;
  const int gw = d.heads * d.dim, vw = d.heads * d.vdim;
  G.oq = 0; G.of = gw; G.ov = 2 * gw;
  y.in = b.stack({{pre + "q", gw}, {pre + "f", gw}, {pre + "v", vw}}, width);
  G.w.bias = b.vec(pre + "f.b", {gw}); G.w.lower = b.vec(pre + "lower", {gw}); G.w.norm = b.vec(pre + "norm", {d.vdim});
  G.out = b.stack({{pre + "o", width}}, vw);
}

void grouped_experts(Builder& b, const Json* c, const std::string& where, const std::string& pre, int width, NetExperts& x)
{
  const Json *r = c->get("router"), *g = r ? r->get("groups") : nullptr;
  const int n = b.integer(r, "experts", where + "router.", 1, EXPERTS_MAX);
  x.top = b.integer(r, "top", where + "router.", 1, std::min(n, EXPERTS_TOP)); x.ff = b.integer(c->get("expert"), "ff", where + "expert.");
  x.groups = b.integer(g, "count", where + "router.groups.", 1, std::min(n, EXPERTS_GROUPS)); x.keep = b.integer(g, "keep", where + "router.groups.", 1, x.groups);
  if (b.rc) return;
  if (n % x.groups || x.top > n / x.groups * x.keep) { b.fail(where + "router.groups: " + std::to_string(x.top) + " of " + std::to_string(n) + " experts from " + std::to_string(x.keep) + " of " + std::to_string(x.groups) + " groups"); return; }
  x.route = ROUTE_SIGMOID; x.gated = false; x.act = LIN_RELU_SQUARED;
  x.router = b.stack({{pre + "router", n}}, width);
  x.correction = b.vec(pre + "correction", {n});
  b.banks(pre, n, x.ff, width, x);
  x.n = n;
}

void build_zenorax(Builder& b, const Json& cfg)
{
  NetSpec& s = b.s;
  const Json* layers = b.layer_list(cfg, false, true);
  if (!layers) return;
  s.embed_scale = b.number(cfg.get("embedding"), "scale", "embedding."); s.logit_cap = b.number(&cfg, "logit_softcap", "");
  const int taps = b.integer(cfg.get("canon"), "taps", "canon.", 1, 64);
  if (!b.rc && !(s.logit_cap > 0.0f)) b.fail("\"logit_softcap\" is not above zero");
  const int L = (int)layers->arr.size(), w = s.width;
  s.rms_final = b.vec("final.norm", {w});
  for (int l = 0; l < L && !b.rc; l++) {
    const Json& c = layers->arr[l];
    const std::string p = "l" + std::to_string(l) + ".", where = "layers[" + std::to_string(l) + "].", type = b.word(&c, "type");
    const Json *mix = c.get("mixer"), *mlp = c.get("mlp");
    NetLayer y;
    y.sandwich = true;
    if (type == "latent_attention") { y.kind = MIX_LATENT; latent_attention(b, mix, where + "mixer.", p + "mix.", w, y); }
    else if (type == "attention") { y.kind = MIX_ATTN; key_value_attention(b, mix, where + "mixer.", p + "mix.", w, y); }
    else if (type == "hgrn2") { y.kind = MIX_GLA; forget_gate_attention(b, mix, where + "mixer.", p + "mix.", w, y); }
    else b.fail("\"" + where + "type\" is not one of latent_attention, attention, hgrn2");
    if (b.rc) return;
    y.rms1 = b.vec(p + "norm1", {w}); y.rms1b = b.vec(p + "norm1b", {w}); y.depth = b.vec(p + "dwa", {l + 2});
    std::vector<float> cw;
    if (!b.floats(p + "canon1", {w, taps}, cw)) return;
    std::vector<float> by_tap(cw.size());
    for (int i = 0; i < w; i++) for (int j = 0; j < taps; j++) by_tap[(size_t)j * w + i] = cw[(size_t)i * taps + j];
    y.conv.taps = taps; y.conv.w = b.upload(by_tap);
    if (mlp && mlp->kind == Json::OBJ) {
      if (b.word(mlp, "kind") != "moe") { b.fail("\"" + where + "mlp.kind\" is not moe"); return; }
      grouped_experts(b, mlp, where + "mlp.", p + "mlp.", w, y.experts);
      if (b.rc) return;
      y.rms2 = b.vec(p + "norm2", {w}); y.rms2b = b.vec(p + "norm2b", {w});
    } else if (mlp && mlp->kind != Json::NUL) b.fail("\"" + where + "mlp\" is neither an object nor null");
    s.layers.push_back(y);
  }
}

struct Arch { const char* name; void (*build)(Builder&, const Json&); };
const Arch ARCHS[] = {{"Samanex", build_samanex}, {"Kiruvik", build_kiruvik}, {"Gamanex", build_gamanex}, {"Zenorax", build_zenorax}};

bool is_dir(const char* path) { struct stat sb; return stat(path, &sb) == 0 && S_ISDIR(sb.st_mode); }

int read_config(const std::string& path, Json& j)
{
  FILE* f = fopen(path.c_str(), "rb");
  if (!f) return set_error(CAI_ERR_INVALID, "model: cannot open %s", path.c_str());
  std::string text; char buf[65536]; size_t k;
  while ((k = fread(buf, 1, sizeof buf, f)) > 0) text.append(buf, k);
  fclose(f);
  std::string err;
  if (!JsonReader::parse(text.data(), text.size(), j, err) || j.kind != Json::OBJ) return set_error(CAI_ERR_INVALID, "model: %s: %s", err.c_str(), path.c_str());
  return CAI_OK;
}

}  // namespace
}  // namespace cai

using namespace cai;

extern "C" int cai_decoder_load(const char* path, int max_tokens, int max_seq, int dtype, cai_decoder_t* out)
{
  CAI_ENTER();
  CAI_REQUIRE(path && out, "cai_decoder_load: null argument");
  *out = nullptr;
  CAI_REQUIRE(dtype == CAI_DTYPE_BF16 || dtype == CAI_DTYPE_F32, "cai_decoder_load: number format %d", dtype);
  if (!is_dir(path)) return cai_decoder_load_gguf(path, max_tokens, max_seq, dtype == CAI_DTYPE_F32 ? CAI_KV_F32 : CAI_KV_F16, out);
  CAI_REQUIRE(max_seq >= 1 && max_seq <= 256 && max_tokens >= 1 && max_tokens <= (1 << 26), "cai_decoder_load: %d sequences, %d tokens", max_seq, max_tokens);
  Json cfg;
  int rc = read_config(std::string(path) + "/config.json", cfg);
  if (rc) return rc;
  const Json* a = cfg.get("architecture");
  const Arch* arch = nullptr; std::string known;
  for (const Arch& k : ARCHS) { if (a && a->kind == Json::STR && a->str == k.name) arch = &k; known += (known.empty() ? "" : ", ") + std::string(k.name); }
  if (!arch) return set_error(CAI_ERR_UNSUPPORTED, "model: architecture \"%s\" is not one of: %s", a && a->kind == Json::STR ? a->str.c_str() : "", known.c_str());
  CAI_READY();
  Builder b;
  if ((rc = b.st.open(std::string(path) + "/model.safetensors"))) return rc;
  arch->build(b, cfg);
  if (b.rc) { net_spec_free(b.s); return b.rc; }
  LayeredNet* n = nullptr;
  if ((rc = net_create(std::move(b.s), max_tokens, max_seq, dtype == CAI_DTYPE_F32 ? ACT_T_F32 : ACT_T_BF16, &n))) return rc;
  return decoder_from_net(n, max_tokens, max_seq, out);
}
