#include "gebuzen_decoder.h"

#include <algorithm>

#include "gebuzen_weight.h"
#include "sequence_cache.h"

namespace lightseq {
namespace hip {

using namespace lsh;

namespace {

constexpr int kFewRows = 64;  // steps of at most this many rows take partial sums from split products
constexpr int kMaxPlanes = 8;
constexpr int kScanRows = 8;  // spans this short run the recurrence token by token

template <typename T>
class Stack : public DecoderStack {
 public:
  Stack(const GebuzenConfig& c, const SafeTensors& file, int slots, int max_step, hipStream_t s)
      : _c(c), _runs(c.runs()), _max_step(max_step), _slots(slots), _stream(s) {
    check();
    _w.load(c, file, s);
    // a layer that is passed through several times has keys and a state of its own in every pass
    _cache.resize(_runs.size());
    for (size_t i = 0; i < _runs.size(); ++i) {
      const GebuzenLayerConfig& l = c.layers[_runs[i].layer];
      _cache[i].k.alloc((size_t)slots * l.kv_heads * max_step * attn_pad(l.dim));
      _cache[i].state.alloc((size_t)slots * l.gla_heads * l.gla_dim * l.gla_vdim);
    }
    CHECK_GPU_ERROR(hipStreamSynchronize(s));
  }

  bool reserve(int rows, int n_seqs, int n_want) override {
    if (rows <= _rows && n_seqs <= _seqs && n_want <= _wants) return false;
    CHECK_GPU_ERROR(hipStreamSynchronize(_stream));
    _rows = std::max(_rows, rows);
    _seqs = std::max(_seqs, n_seqs);
    _wants = std::max(_wants, n_want);
    const size_t R = _rows, W = _c.width;
    size_t proj = 0, low = 0, q = 0, left = 0, right = 0, chunk = 0, act = 0, dec = 0;
    for (size_t i = 0; i < _c.layers.size(); ++i) {
      const GebuzenLayerConfig& l = _c.layers[i];
      const AttnShape a = attn_shape(l);
      const GlaShape g = gla_shape(i);
      proj = std::max(proj, (size_t)_w.layers[i].t_cols);
      low = std::max(low, (size_t)g.rank);
      q = std::max(q, (size_t)l.heads * a.dim_pad);
      left = std::max(left, (size_t)l.heads * l.dim);
      right = std::max(right, (size_t)l.gla_heads * l.gla_vdim);
      dec = std::max(dec, attn_decode_workspace(std::min(_rows, _slots), a));
      if (gla_chunked_supported(g, _w.layers[i].t_cols))
        chunk = std::max(chunk, gla_chunked_workspace(_rows, _seqs, g));
      act = std::max(act, (size_t)l.ff);
    }
    const size_t few = std::min(_rows, kFewRows) * W * kMaxPlanes;
    const size_t many = _rows > kFewRows ? R * W : 0;
    _x.alloc(R * W);
    _h.alloc(R * W);
    _hf.alloc((size_t)_wants * W);
    _proj.alloc(R * proj);
    _low.alloc(R * low);
    _q.alloc(R * q);
    _left.alloc(R * left);
    _right.alloc(R * right);
    _chunk.alloc(chunk);
    _attn_ws.alloc(dec);
    _act.alloc(R * act);
    for (int i = 0; i < 2; ++i) {
      _yf[i].alloc(few);
      _y[i].alloc(many);
    }
    _logits.alloc((size_t)_wants * _c.vocab);
    return true;
  }

  const float* run(const StepBatch& b, const StepTaps& taps, int tap_step) override {
    const int R = b.rows, W = _c.width, n = (int)_runs.size();
    const bool few = R <= kFewRows;
    const bool all_wanted = b.n_want > 0 && b.want == nullptr;
    const float eps = (float)_c.eps;
    LSH_CALL(lm_norm<T>(_x.get(), AddSpec{}, norm1(0), _h.get(), R, W, eps, b.ids, _w.embed.get(),
                        _c.vocab, nullptr, b.zero_flag, b.zero_flag ? 1 : 0, _stream,
                        ahead_of(0, b)));
    for (int i = 0; i < n; ++i) {
      const GebuzenLayerConfig& l = _c.layers[_runs[i].layer];
      const GebuzenLayerWeight<T>& w = _w.layers[_runs[i].layer];
      // the norm that reads the stream after this layer
      NormSpec next;
      T* next_out = _h.get();
      if (i + 1 < n) {
        next = norm1(i + 1);
      } else if (all_wanted) {
        next = rms(_w.final_norm);
        next_out = _hf.get();
      }
      mixer(i, b);
      AddSpec add = spec(few, 0.5f * (float)_c.residual_mult);
      products_out(l, w, R, few, add);
      add.post_w = w.left_norm.get();
      add.second.post_w = w.right_norm.get();
      if (l.ff) {
        LSH_CALL(lm_norm<T>(_x.get(), add, rms(w.norm2), _h.get(), R, W, eps, nullptr, nullptr, 0,
                            nullptr, nullptr, 0, _stream));
        LSH_CALL(gemm_gated<T>(_h.get(), W, w.up.get(), _act.get(), l.ff, R, l.ff, W, kGateRelu,
                               _stream));
        add = spec(few, (float)_c.residual_mult);
        product_down(l, w, R, few, add);
      }
      InjectSpec inject = i + 1 < n ? ahead_of(i + 1, b) : InjectSpec{};
      if (inject.any() && taps.wants(i, tap_step, "res_out")) {
        // the stream between this layer and what comes ahead of the next one has to be seen
        LSH_CALL(lm_norm<T>(_x.get(), add, NormSpec{}, nullptr, R, W, eps, nullptr, nullptr, 0,
                            nullptr, nullptr, 0, _stream));
        taps.copy(i, tap_step, "res_out", _x.get(), (size_t)R * W * sizeof(float), _stream);
        add = AddSpec{};
      }
      LSH_CALL(lm_norm<T>(_x.get(), add, next, next_out, R, W, eps, nullptr, _w.embed.get(),
                          _c.vocab, nullptr, nullptr, 0, _stream, inject));
      if (!inject.any())
        taps.copy(i, tap_step, "res_out", _x.get(), (size_t)R * W * sizeof(float), _stream);
    }
    if (b.n_want == 0) return _logits.get();
    if (!all_wanted)
      LSH_CALL(lm_norm<T>(_x.get(), AddSpec{}, rms(_w.final_norm), _hf.get(), b.n_want, W, eps,
                          nullptr, nullptr, 0, b.want, nullptr, 0, _stream));
    GemmEpilogue scaled;
    scaled.scale = (float)_c.logit_scale;
    LSH_CALL((gemm_float<T, float>(_hf.get(), W, _w.head.get(), _logits.get(), _c.vocab, nullptr, 0,
                                   _c.vocab, b.n_want, _c.vocab, W, _stream, scaled)));
    return _logits.get();
  }

 private:
  void check() const {
    for (const GebuzenLayerConfig& l : _c.layers)
      if (l.dim > 256 || l.gla_dim > 256 || l.gla_vdim > 256)
        throw std::runtime_error("config: head sizes above 256 are not supported");
    if (_c.width > 8192 || (_c.width > 4096 && _c.width % 4))
      throw std::runtime_error("config: width above 8192 is not supported");
  }
  AttnShape attn_shape(const GebuzenLayerConfig& l) const {
    return AttnShape{l.heads, l.kv_heads, l.dim, l.dim, attn_pad(l.dim), attn_pad(l.dim), _max_step};
  }
  GlaShape gla_shape(size_t layer) const {
    const GebuzenLayerConfig& l = _c.layers[layer];
    const GebuzenLayerWeight<T>& w = _w.layers[layer];
    return GlaShape{l.gla_heads, l.gla_dim, l.gla_vdim, w.rank,    w.gq_col,
                    w.gk_col,    w.gv_col,  w.gg_col,   (float)(1.0 / l.tau), (float)_c.eps};
  }
  static NormSpec rms(const DeviceBuffer<float>& w) { return NormSpec{w.get(), nullptr, kRmsNorm}; }
  NormSpec norm1(int i) const { return rms(_w.layers[_runs[i].layer].norm1); }
  // what is added to the stream ahead of a run
  InjectSpec ahead_of(int i, const StepBatch& b) const {
    InjectSpec in;
    if (_runs[i].again) in.ids = b.ids;
    if (_runs[i].step >= 0) in.vec = _w.loop_step.get() + (size_t)_runs[i].step * _c.width;
    return in;
  }
  static AddSpec spec(bool few, float scale) {
    AddSpec add;
    add.y_is_float = few;
    add.scale = scale;
    add.post_kind = kRmsNorm;
    return add;
  }

  // _h -> _left, _right
  void mixer(int i, const StepBatch& b) {
    const int layer = _runs[i].layer;
    const GebuzenLayerConfig& l = _c.layers[layer];
    const GebuzenLayerWeight<T>& w = _w.layers[layer];
    LayerCache<T>& c = _cache[i];
    const int R = b.rows, ld = w.t_cols;
    GemmEpilogue biased;
    biased.bias = w.in_bias.get();
    LSH_CALL((gemm_float<T, T>(_h.get(), _c.width, w.in.get(), _proj.get(), ld, _low.get(), w.rank,
                               w.t_cols, R, w.in_cols, _c.width, _stream, biased)));
    const AttnShape sh = attn_shape(l);
    AttnMask mask{0, 0, (float)l.scale, true};
    mask.chunk = l.chunk;
    mask.sinks = w.sink.get();
    const GlaShape gs = gla_shape(layer);
    const GlaWeights gw{w.a2.get(), w.a2_bias.get(), w.head_norm.get()};
    const bool one = b.max_n == 1;
    if (one && attn_decode_append_supported(sh, w.q_col, w.k_col, ld)) {
      LSH_CALL(attn_decode_append<T>(_proj.get(), ld, w.q_col, w.k_col, c.k.get(), _left.get(),
                                     b.row_slot, b.row_pos, R, b.max_len, _attn_ws.get(), sh, mask,
                                     _stream));
    } else {
      LSH_CALL(attn_prepare<T>(_proj.get(), ld, w.q_col, w.k_col, -1, nullptr, nullptr, 0.f, nullptr,
                               0, _q.get(), c.k.get(), nullptr, b.row_slot, b.row_pos, R, sh,
                               _stream));
      if (one)
        LSH_CALL(attn_decode<T>(_q.get(), c.k.get(), c.k.get(), nullptr, 0, -1, _left.get(),
                                b.row_slot, b.row_pos, R, b.max_len, _attn_ws.get(), sh, mask,
                                _stream));
      else
        LSH_CALL(attn_prefill<T>(_q.get(), c.k.get(), c.k.get(), nullptr, 0, -1, _left.get(), b.spans,
                                 b.n_seqs, b.max_n, sh, mask, _stream));
    }
    if (one)
      LSH_CALL(gla_step<T>(_proj.get(), ld, _low.get(), gw, c.state.get(), _right.get(), b.row_slot,
                           b.row_pos, R, gs, _stream));
    else if (b.max_n > kScanRows && gla_chunked_supported(gs, ld))
      LSH_CALL(gla_chunked<T>(_proj.get(), ld, _low.get(), gw, c.state.get(), _right.get(),
                              _chunk.get(), b.spans, b.n_seqs, b.max_n, R, gs, _stream));
    else
      LSH_CALL(gla_scan<T>(_proj.get(), ld, _low.get(), gw, c.state.get(), _right.get(), b.spans,
                           b.n_seqs, gs, _stream));
  }

  // both mixers' output projections: what is left to add to the stream
  void products_out(const GebuzenLayerConfig& l, const GebuzenLayerWeight<T>& w, int R, bool few,
                    AddSpec& add) {
    const int k0 = l.heads * l.dim, k1 = l.gla_heads * l.gla_vdim;
    if (few) {
      add.part_stride = add.second.part_stride = (long)R * _c.width;
      LSH_CALL(gemm_float_planes2<T>(FloatProduct<T>{_left.get(), k0, w.left_o.get(), _yf[0].get(), k0},
                                     FloatProduct<T>{_right.get(), k1, w.right_o.get(), _yf[1].get(), k1},
                                     R, _c.width, kMaxPlanes, &add.parts, &add.second.parts, _stream));
    } else {
      add.parts = add.second.parts = 1;
      many_rows(_left, k0, w.left_o, R, 0);
      many_rows(_right, k1, w.right_o, R, 1);
    }
    locate(few, 0, add);
    locate(few, 1, add.second);
  }
  // the feed-forward's
  void product_down(const GebuzenLayerConfig& l, const GebuzenLayerWeight<T>& w, int R, bool few,
                    AddSpec& add) {
    add.parts = 1;
    if (few) {
      add.part_stride = (long)R * _c.width;
      LSH_CALL(gemm_float_planes<T>(_act.get(), l.ff, w.down.get(), _yf[0].get(), R, _c.width, l.ff,
                                    kMaxPlanes, &add.parts, _stream));
    } else {
      many_rows(_act, l.ff, w.down, R, 0);
    }
    locate(few, 0, add);
  }
  void many_rows(const DeviceBuffer<T>& a, int k, const DeviceBuffer<T>& w, int R, int which) {
    const int W = _c.width;
    LSH_CALL((gemm_float<T, T>(a.get(), k, w.get(), _y[which].get(), W, nullptr, 0, W, R, W, k,
                               _stream)));
  }
  void locate(bool few, int which, AddPart& part) {
    part.row_stride = _c.width;
    part.y = few ? (const void*)_yf[which].get() : (const void*)_y[which].get();
  }

  const GebuzenConfig _c;
  const std::vector<GebuzenLayerRun> _runs;
  const int _max_step, _slots;
  hipStream_t _stream;
  GebuzenWeight<T> _w;
  std::vector<LayerCache<T>> _cache;  // per run
  int _rows = 0, _seqs = 0, _wants = 0;
  DeviceBuffer<float> _x, _low, _chunk, _attn_ws, _yf[2], _logits;
  DeviceBuffer<T> _h, _hf, _proj, _q, _left, _right, _act, _y[2];
};

}  // namespace

std::unique_ptr<DecoderStack> create_gebuzen_stack(const GebuzenConfig& config,
                                                   const SafeTensors& file, bool float32, int slots,
                                                   int max_step, hipStream_t stream) {
  if (float32) return std::make_unique<Stack<float>>(config, file, slots, max_step, stream);
  return std::make_unique<Stack<bf16_t>>(config, file, slots, max_step, stream);
}

}  // namespace hip
}  // namespace lightseq
