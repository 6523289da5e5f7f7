#include "gebuzen_weight.h"

#include "stacked_weight.h"

namespace lightseq {
namespace hip {

template <typename T>
void GebuzenWeight<T>::load(const GebuzenConfig& c, const SafeTensors& f, hipStream_t s) {
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
  final_norm = floats("final.norm", {W});
  if (c.loop_times) loop_step = floats("loop.step", {c.loop_times, W});
  layers.clear();
  layers.resize(c.layers.size());
  for (size_t i = 0; i < c.layers.size(); ++i) {
    const GebuzenLayerConfig& l = c.layers[i];
    GebuzenLayerWeight<T>& d = layers[i];
    const std::string p = "l" + std::to_string(i) + ".", left = p + "mix.left.",
                      right = p + "mix.right.";
    const long q = (long)l.heads * l.dim, k = (long)l.kv_heads * l.dim;
    const long gk = (long)l.gla_heads * l.gla_dim, gv = (long)l.gla_heads * l.gla_vdim;
    d.norm1 = floats(p + "norm1", {W});
    Stacked<T> in;
    Stacked<float> bias;
    long at = 0;
    const auto section = [&](const std::string& name, long rows, bool biased) {
      const long first = at, pad = (8 - rows % 8) % 8;
      in.add(f, name, {rows, W});
      in.add_zeros(pad * W);
      if (biased) bias.add(f, name + ".b", {rows});
      else bias.add_zeros(rows);
      bias.add_zeros(pad);
      at += rows + pad;
      return (int)first;
    };
    d.q_col = section(left + "q", q, true);
    d.k_col = section(left + "k", k, true);
    d.gq_col = section(right + "q", gk, false);
    d.gk_col = section(right + "k", gk, false);
    d.gv_col = section(right + "v", gv, false);
    d.gg_col = section(right + "g", gv, false);
    d.t_cols = (int)at;
    const SafeTensors::Tensor& a1 = f.get(right + "a1");
    const long rank = a1.shape.empty() ? 0 : a1.shape[0];
    if (rank <= 0) throw std::runtime_error("tensor '" + right + "a1' has no rows");
    d.rank = (int)((rank + 15) / 16 * 16);
    in.add(f, right + "a1", {rank, W});
    in.add_zeros((d.rank - rank) * W);
    bias.add_zeros(d.rank);
    d.in_cols = d.t_cols + d.rank;
    d.in = in.upload(s);
    d.in_bias = bias.upload(s);
    d.sink = floats(left + "sink", {l.heads});
    Stacked<float> a2;
    a2.add_rows(f, right + "a2", gk, rank, d.rank);
    d.a2 = a2.upload(s);
    d.a2_bias = floats(right + "a2.b", {gk});
    d.head_norm = floats(right + "norm", {l.gla_vdim});
    d.left_o = matrix(left + "o", W, q);
    d.right_o = matrix(right + "o", W, gv);
    d.left_norm = floats(left + "out", {W});
    d.right_norm = floats(right + "out", {W});
    if (l.ff) {
      d.norm2 = floats(p + "norm2", {W});
      Stacked<T> up;
      up.add(f, p + "mlp.gate", {l.ff, W});
      up.add(f, p + "mlp.up", {l.ff, W});
      d.up = up.upload(s);
      d.down = matrix(p + "mlp.down", W, l.ff);
    }
  }
}

template struct GebuzenWeight<float>;
template struct GebuzenWeight<bf16_t>;

}  // namespace hip
}  // namespace lightseq
