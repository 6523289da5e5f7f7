#include "sudevik_config.h"

#include <algorithm>
#include <cmath>

namespace lightseq {
namespace hip {

std::vector<double> RotaryConfig::frequencies(double* magnitude) const {
  std::vector<double> f(dims / 2);
  for (int i = 0; i < dims / 2; ++i) f[i] = std::pow(base, -2.0 * i / dims);
  *magnitude = 1.0;
  if (!scaled) return f;
  // the pair index whose wave turns t times within the original length
  const auto pair_of = [&](double t) {
    return dims * std::log(original / (2 * M_PI * t)) / (2 * std::log(base));
  };
  const double lo = std::max(std::floor(pair_of(fast)), 0.0);
  const double hi = std::min(std::ceil(pair_of(slow)), dims - 1.0);
  for (int i = 0; i < dims / 2; ++i) {
    const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
    f[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp);
  }
  *magnitude = 0.1 * std::log(factor) + 1.0;
  return f;
}

SudevikConfig SudevikConfig::parse(const Json& c) {
  SudevikConfig out;
  out.vocab = c.positive("vocab");
  out.width = c.positive("width");
  out.eps = c.at("norm").at("eps").number();
  for (const Json& e : c.at("layers").items()) {
    SudevikLayerConfig l;
    const int index = (int)out.layers.size();
    const std::string type = e.at("type").string();
    const Json& m = e.at("mixer");
    l.heads = m.positive("heads");
    l.kv_heads = m.positive("kv_heads");
    l.dim = m.positive("dim");
    l.vdim = m.positive("vdim");
    if (l.heads % l.kv_heads) throw std::runtime_error("config: heads must be a multiple of kv_heads");
    if (type == "attention") {
      l.attention = true;
      l.scale = m.at("scale").number();
      const Json& rot = m["rot"];
      if (!rot.is_null()) {
        l.rot.dims = rot.positive("dims");
        l.rot.base = rot.at("base").number();
        if (l.rot.dims % 2 || l.rot.dims > l.dim)
          throw std::runtime_error("config: rot.dims must be even and at most dim");
        const Json& sc = rot["scaling"];
        if (!sc.is_null()) {
          l.rot.scaled = true;
          l.rot.factor = sc.at("factor").number();
          l.rot.original = sc.at("original").number();
          l.rot.fast = sc.at("fast").number();
          l.rot.slow = sc.at("slow").number();
        }
      }
      const Json& mask = m["mask"];
      if (!mask.is_null()) {
        l.window = mask.positive("size");
        if (!mask["keep_first"].is_null()) l.keep_first = (int)mask["keep_first"].integer();
      }
      if (!m["kv_from"].is_null()) {
        l.kv_from = (int)m["kv_from"].integer();
        if (l.kv_from < 0 || l.kv_from >= index || !out.layers[l.kv_from].attention ||
            out.layers[l.kv_from].kv_from >= 0)
          throw std::runtime_error("config: kv_from must name an earlier layer with keys of its own");
        const SudevikLayerConfig& src = out.layers[l.kv_from];
        if (src.kv_heads != l.kv_heads || src.dim != l.dim || src.vdim != l.vdim)
          throw std::runtime_error("config: kv_from names a layer of other head sizes");
      }
    } else if (type == "delta") {
      l.taps = m.positive("conv");
    } else {
      throw std::runtime_error("config: unknown layer type '" + type + "'");
    }
    const Json& f = e["mlp"];
    if (!f.is_null()) {
      if (f.at("kind").string() != "moe")
        throw std::runtime_error("config: unknown mlp kind '" + f.at("kind").string() + "'");
      l.ff = f.at("expert").positive("ff");
      l.experts = f.at("router").positive("experts");
      l.top = f.at("router").positive("top");
      if (l.top > l.experts) throw std::runtime_error("config: more choices than experts");
    }
    out.layers.push_back(l);
  }
  if (out.layers.empty()) throw std::runtime_error("config: no layers");
  return out;
}

}  // namespace hip
}  // namespace lightseq
