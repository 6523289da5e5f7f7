#include "gebuzen_config.h"

namespace lightseq {
namespace hip {

GebuzenConfig GebuzenConfig::parse(const Json& c) {
  GebuzenConfig out;
  out.vocab = c.positive("vocab");
  out.width = c.positive("width");
  out.eps = c.at("norm").at("eps").number();
  out.residual_mult = c.at("residual_mult").number();
  out.logit_scale = c.at("logit_scale").number();
  for (const Json& e : c.at("layers").items()) {
    GebuzenLayerConfig l;
    const std::string type = e.at("type").string();
    if (type != "parallel") throw std::runtime_error("config: unknown layer type '" + type + "'");
    const Json &left = e.at("mixer").at("left"), &right = e.at("mixer").at("right");
    l.heads = left.positive("heads");
    l.kv_heads = left.positive("kv_heads");
    l.dim = left.positive("dim");
    if (l.heads % l.kv_heads) throw std::runtime_error("config: heads must be a multiple of kv_heads");
    if (left.positive("vdim") != l.dim)
      throw std::runtime_error("config: the values are the keys: vdim must be dim");
    l.scale = left.at("scale").number();
    if (!left["mask"].is_null()) l.chunk = left["mask"].positive("size");
    l.gla_heads = right.positive("heads");
    l.gla_dim = right.positive("dim");
    l.gla_vdim = right.positive("vdim");
    l.tau = right.at("tau").number();
    if (!(l.tau > 0)) throw std::runtime_error("config: 'tau' must be positive");
    const Json& f = e["mlp"];
    if (!f.is_null()) {
      if (f.at("kind").string() != "dense")
        throw std::runtime_error("config: unknown mlp kind '" + f.at("kind").string() + "'");
      l.ff = f.positive("ff");
    }
    out.layers.push_back(l);
  }
  if (out.layers.empty()) throw std::runtime_error("config: no layers");
  const Json& loop = c["loop"];
  if (!loop.is_null()) {
    out.loop_start = (int)loop.at("start").integer();
    out.loop_stop = (int)loop.at("stop").integer();
    out.loop_times = loop.positive("times");
    if (out.loop_start < 0 || out.loop_start >= out.loop_stop ||
        out.loop_stop > (int)out.layers.size())
      throw std::runtime_error("config: the loop must name a run of layers");
  }
  return out;
}

std::vector<GebuzenLayerRun> GebuzenConfig::runs() const {
  std::vector<GebuzenLayerRun> out;
  const auto range = [&](int from, int to) {
    for (int i = from; i < to; ++i) {
      out.emplace_back();
      out.back().layer = i;
    }
  };
  const int n = (int)layers.size();
  if (loop_times == 0) {
    range(0, n);
    return out;
  }
  range(0, loop_start);
  for (int t = 0; t < loop_times; ++t) {
    const size_t first = out.size();
    range(loop_start, loop_stop);
    out[first].step = t;
    out[first].again = t > 0;
  }
  range(loop_stop, n);
  return out;
}

}  // namespace hip
}  // namespace lightseq
