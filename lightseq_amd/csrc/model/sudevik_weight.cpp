#include "sudevik_weight.h"

#include "stacked_weight.h"

namespace lightseq {
namespace hip {

using lsh::bf16_t;

template <typename T>
void SudevikWeight<T>::load(const SudevikConfig& c, const SafeTensors& f, hipStream_t s) {
  const long W = c.width, V = c.vocab;
  const auto floats = [&](const std::string& name, const std::vector<long>& shape) {
    Stacked<float> st;
    st.add(f, name, shape);
    return st.upload(s);
  };
  const auto matrix = [&](const std::string& name, long rows, long cols) {
    Stacked<T> st;
    st.add(f, name, {rows, cols});
    return st.upload(s);
  };
  embed = matrix("embed", V, W);
  head = matrix("head", V, W);
  final_w = floats("final.norm", {W});
  final_b = floats("final.norm.b", {W});
  layers.clear();
  layers.resize(c.layers.size());
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const SudevikLayerConfig& l = c.layers[i];
    SudevikLayerWeight<T>& d = layers[i];
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.";
    const long q = (l.attention ? l.heads : l.kv_heads) * (long)l.dim;
    const long k = (long)l.kv_heads * l.dim, ctx = (long)l.heads * l.vdim;
    const long v = l.attention ? (long)l.kv_heads * l.vdim : ctx;
    const char* norms[4] = {"norm1", "norm1b", "norm2", "norm2b"};
    for (int n = 0; n < (l.experts ? 4 : 2); ++n) {
      d.norm_w[n] = floats(p + norms[n], {W});
      d.norm_b[n] = floats(p + norms[n] + ".b", {W});
    }
    Stacked<T> in;
    in.add(f, m + "q", {q, W});
    long at = q;
    if (l.kv_from < 0) {
      in.add(f, m + "k", {k, W});
      in.add(f, m + "v", {v, W});
      d.k_col = (int)at;
      d.v_col = (int)(at + k);
      at += k + v;
    }
    in.add(f, m + "g", {ctx, W});
    d.g_col = (int)at;
    at += ctx;
    d.t_cols = (int)at;
    if (!l.attention) {
      in.add(f, m + "b", {l.heads, W});
      in.add(f, m + "a", {l.heads, W});
      at += 2L * l.heads;
    }
    d.in_cols = (int)at;
    d.in = in.upload(s);
    d.out = matrix(m + "o", W, ctx);
    if (l.attention) {
      d.q_norm = floats(m + "q.norm", {l.dim});
      if (l.kv_from < 0) d.k_norm = floats(m + "k.norm", {l.dim});
    } else {
      Stacked<float> conv;
      conv.add(f, m + "q.conv", {q, l.taps});
      conv.add(f, m + "k.conv", {k, l.taps});
      conv.add(f, m + "v.conv", {v, l.taps});
      d.conv = conv.upload(s);
      d.a_log = floats(m + "A_log", {l.heads});
      d.dt_bias = floats(m + "dt_bias", {l.heads});
      d.head_norm = floats(m + "norm", {l.vdim});
    }
    if (l.experts) {
      const std::string e = p + "mlp.";
      d.router = matrix(e + "router", l.experts, W);
      d.router_b = floats(e + "router.b", {l.experts});
      Stacked<T> up, down;
      for (int x = 0; x < l.experts; ++x) {
        const std::string ex = e + "e" + std::to_string(x) + ".";
        up.add(f, ex + "gate", {l.ff, W});
        up.add(f, ex + "up", {l.ff, W});
        down.add(f, ex + "down", {W, l.ff});
      }
      d.up = up.upload(s);
      d.down = down.upload(s);
    }
  }
}

template struct SudevikWeight<float>;
template struct SudevikWeight<bf16_t>;

}  // namespace hip
}  // namespace lightseq
