#include "sudevik_decoder.h"

#include <algorithm>
#include <cmath>

#include "sequence_cache.h"
#include "sudevik_weight.h"

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
  Stack(const SudevikConfig& c, const SafeTensors& file, int slots, int max_step, hipStream_t s)
      : _c(c), _max_step(max_step), _slots(slots), _stream(s) {
    check();
    _w.load(c, file, s);
    _cache.resize(c.layers.size());
    _rot.resize(c.layers.size(), -1);
    for (size_t i = 0; i < c.layers.size(); ++i) {
      const SudevikLayerConfig& l = c.layers[i];
      LayerCache<T>& k = _cache[i];
      if (l.attention) {
        if (l.kv_from < 0) {
          const size_t n = (size_t)slots * l.kv_heads * max_step;
          k.k.alloc(n * attn_pad(l.dim));
          k.v.alloc(n * attn_pad(l.vdim));
        }
        if (l.rot.dims) _rot[i] = rotation_table(l.rot);
      } else {
        const DeltaShape d = delta_shape(l);
        k.conv.alloc((size_t)slots * d.taps * d.channels());
        k.state.alloc((size_t)slots * d.heads * d.dim * d.vdim);
      }
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
    size_t proj = 0, ba = 0, q = 0, ctx = 0, dqk = 0, dv = 0, dh = 0, chunk = 0, E = 0, top = 0,
           act = 0, dec = 0;
    for (size_t i = 0; i < _c.layers.size(); ++i) {
      const SudevikLayerConfig& l = _c.layers[i];
      proj = std::max(proj, (size_t)ld_of(_w.layers[i]));
      ctx = std::max(ctx, (size_t)l.heads * l.vdim);
      if (l.attention) {
        const AttnShape a = attn_shape(l);
        q = std::max(q, (size_t)l.heads * a.dim_pad);
        dec = std::max(dec, attn_decode_workspace(std::min(_rows, _slots), a));
      } else {
        const DeltaShape d = delta_shape(l);
        ba = std::max(ba, 2 * (size_t)l.heads);
        dqk = std::max(dqk, (size_t)l.kv_heads * l.dim);
        dv = std::max(dv, (size_t)l.heads * l.vdim);
        dh = std::max(dh, (size_t)l.heads);
        if (delta_chunked_supported(d))
          chunk = std::max(chunk, delta_chunked_workspace(_rows, _seqs, d));
      }
      E = std::max(E, (size_t)l.experts);
      top = std::max(top, (size_t)l.top);
      act = std::max(act, (size_t)l.top * l.ff);
    }
    const bool many = _rows > kFewRows;
    _x.alloc(R * W);
    _h.alloc(R * W);
    _hf.alloc((size_t)_wants * W);
    _proj.alloc(R * proj);
    _ba.alloc(R * ba);
    _q.alloc(R * q);
    _ctx.alloc(R * ctx);
    _dq.alloc(R * dqk);
    _dk.alloc(R * dqk);
    _dv.alloc(R * dv);
    _do.alloc(R * dv);
    _dg.alloc(R * dh);
    _dbeta.alloc(R * dh);
    _chunk.alloc(chunk);
    _attn_ws.alloc(dec);
    _yf.alloc((size_t)std::min(_rows, kFewRows) * W * kMaxPlanes);
    _y.alloc(many ? R * W : 0);
    _router.alloc(R * E);
    _weight.alloc(R * top);
    _count.alloc(E);
    _list.alloc(R * E);
    _act.alloc(R * act);
    _exf.alloc((size_t)std::min(_rows, kFewRows) * top * W);
    _ex.alloc(many ? R * top * W : 0);
    _logits.alloc((size_t)_wants * _c.vocab);
    return true;
  }

  const float* run(const StepBatch& b, const StepTaps& taps, int tap_step) override {
    const int R = b.rows, W = _c.width, n = (int)_c.layers.size();
    const bool few = R <= kFewRows;
    const bool all_wanted = b.n_want > 0 && b.want == nullptr;
    const float eps = (float)_c.eps;
    NormSpec first{_w.layers[0].norm_w[0].get(), _w.layers[0].norm_b[0].get()};
    LSH_CALL(lm_norm<T>(_x.get(), AddSpec{}, first, _h.get(), R, W, eps, b.ids, _w.embed.get(),
                        _c.vocab, nullptr, b.zero_flag, b.zero_flag ? 1 : 0, _stream));
    for (int i = 0; i < n; ++i) {
      const SudevikLayerConfig& l = _c.layers[i];
      const SudevikLayerWeight<T>& w = _w.layers[i];
      // the norm that reads the stream after this layer
      NormSpec next;
      T* next_out = _h.get();
      if (i + 1 < n) {
        next = NormSpec{_w.layers[i + 1].norm_w[0].get(), _w.layers[i + 1].norm_b[0].get()};
      } else if (all_wanted) {
        next = NormSpec{_w.final_w.get(), _w.final_b.get()};
        next_out = _hf.get();
      }
      mixer(i, b);
      AddSpec add = project_out(w, l.heads * l.vdim, R, few);
      add.post_w = w.norm_w[1].get();
      add.post_b = w.norm_b[1].get();
      if (l.experts) {
        const NormSpec inner{w.norm_w[2].get(), w.norm_b[2].get()};
        LSH_CALL(lm_norm<T>(_x.get(), add, inner, _h.get(), R, W, eps, nullptr, nullptr, 0, nullptr,
                            _count.get(), l.experts, _stream));
        add = experts(l, w, R, few);
        add.post_w = w.norm_w[3].get();
        add.post_b = w.norm_b[3].get();
      }
      LSH_CALL(lm_norm<T>(_x.get(), add, next, next_out, R, W, eps, nullptr, nullptr, 0, nullptr,
                          nullptr, 0, _stream));
      taps.copy(i, tap_step, "res_out", _x.get(), (size_t)R * W * sizeof(float), _stream);
    }
    if (b.n_want == 0) return _logits.get();
    if (!all_wanted) {
      const NormSpec fin{_w.final_w.get(), _w.final_b.get()};
      LSH_CALL(lm_norm<T>(_x.get(), AddSpec{}, fin, _hf.get(), b.n_want, W, eps, nullptr, nullptr, 0,
                          b.want, nullptr, 0, _stream));
    }
    LSH_CALL((gemm_float<T, float>(_hf.get(), W, _w.head.get(), _logits.get(), _c.vocab, nullptr, 0,
                                   _c.vocab, b.n_want, _c.vocab, W, _stream)));
    return _logits.get();
  }

 private:
  void check() const {
    for (const SudevikLayerConfig& l : _c.layers) {
      if (l.dim > 256 || l.vdim > 256)
        throw std::runtime_error("config: head sizes above 256 are not supported");
      if (l.taps > 16)
        throw std::runtime_error("config: convolutions of more than 16 taps are not supported");
      if (l.experts > 1024 || l.top > 64)
        throw std::runtime_error("config: at most 64 choices of at most 1024 experts are supported");
    }
    if (_c.width > 8192 || (_c.width > 4096 && _c.width % 4))
      throw std::runtime_error("config: width above 8192 is not supported");
  }
  static int ld_of(const SudevikLayerWeight<T>& w) { return (w.t_cols + 7) & ~7; }
  AttnShape attn_shape(const SudevikLayerConfig& l) const {
    return AttnShape{l.heads, l.kv_heads, l.dim, l.vdim, attn_pad(l.dim), attn_pad(l.vdim), _max_step};
  }
  static DeltaShape delta_shape(const SudevikLayerConfig& l) {
    return DeltaShape{l.heads, l.kv_heads, l.dim, l.vdim, l.taps};
  }

  // table of cosines and sines for every position, shared by layers that rotate alike
  int rotation_table(const RotaryConfig& r) {
    for (size_t i = 0; i < _tables.size(); ++i)
      if (_tables[i].first == r) return (int)i;
    double mag = 1;
    const std::vector<double> f = r.frequencies(&mag);
    std::vector<float2> t((size_t)_max_step * f.size());
    for (int p = 0; p < _max_step; ++p)
      for (size_t i = 0; i < f.size(); ++i)
        t[(size_t)p * f.size() + i] =
            make_float2((float)(mag * std::cos(p * f[i])), (float)(mag * std::sin(p * f[i])));
    _tables.emplace_back(r, DeviceBuffer<float2>(t.size()));
    _tables.back().second.upload(t.data(), t.size(), _stream);
    CHECK_GPU_ERROR(hipStreamSynchronize(_stream));
    return (int)_tables.size() - 1;
  }

  // _h -> _ctx
  void mixer(int i, const StepBatch& b) {
    const SudevikLayerConfig& l = _c.layers[i];
    const SudevikLayerWeight<T>& w = _w.layers[i];
    const int R = b.rows, ld = ld_of(w);
    const float eps = (float)_c.eps;
    LSH_CALL((gemm_float<T, T>(_h.get(), _c.width, w.in.get(), _proj.get(), ld, _ba.get(),
                               2L * l.heads, w.t_cols, R, w.in_cols, _c.width, _stream)));
    if (l.attention) {
      const AttnShape sh = attn_shape(l);
      LayerCache<T>& kv = _cache[l.kv_from < 0 ? i : l.kv_from];
      const float2* table = _rot[i] < 0 ? nullptr : _tables[_rot[i]].second.get();
      LSH_CALL(attn_prepare<T>(_proj.get(), ld, w.q_col, w.k_col, w.v_col, w.q_norm.get(),
                               w.k_norm.get(), eps, table, l.rot.dims / 2, _q.get(), kv.k.get(),
                               kv.v.get(), b.row_slot, b.row_pos, R, sh, _stream));
      const AttnMask mask{l.window, l.keep_first, (float)l.scale, true};
      if (b.max_n == 1)
        LSH_CALL(attn_decode<T>(_q.get(), kv.k.get(), kv.v.get(), _proj.get(), ld, w.g_col,
                                _ctx.get(), b.row_slot, b.row_pos, R, b.max_len, _attn_ws.get(), sh,
                                mask, _stream));
      else
        LSH_CALL(attn_prefill<T>(_q.get(), kv.k.get(), kv.v.get(), _proj.get(), ld, w.g_col,
                                 _ctx.get(), b.spans, b.n_seqs, b.max_n, sh, mask, _stream));
      return;
    }
    const DeltaShape sh = delta_shape(l);
    LayerCache<T>& c = _cache[i];
    if (b.max_n == 1) {
      LSH_CALL(delta_step<T>(_proj.get(), ld, w.g_col, _ba.get(), w.conv.get(), w.a_log.get(),
                             w.dt_bias.get(), w.head_norm.get(), eps, c.conv.get(), c.state.get(),
                             _ctx.get(), b.row_slot, b.row_pos, R, sh, _stream));
      return;
    }
    LSH_CALL(delta_prepare<T>(_proj.get(), ld, _ba.get(), w.conv.get(), w.a_log.get(),
                              w.dt_bias.get(), c.conv.get(), _dq.get(), _dk.get(), _dv.get(),
                              _dg.get(), _dbeta.get(), b.spans, b.n_seqs, b.max_n, sh, _stream));
    if (b.max_n > kScanRows && delta_chunked_supported(sh))
      LSH_CALL(delta_chunked<T>(_dq.get(), _dk.get(), _dv.get(), _dg.get(), _dbeta.get(),
                                c.state.get(), _do.get(), _chunk.get(), b.spans, b.n_seqs, b.max_n,
                                R, sh, _stream));
    else
      LSH_CALL(delta_scan<T>(_dq.get(), _dk.get(), _dv.get(), _dg.get(), _dbeta.get(),
                             c.state.get(), _do.get(), b.spans, b.n_seqs, sh, _stream));
    LSH_CALL(delta_gated_norm<T>(_do.get(), _proj.get(), ld, w.g_col, w.head_norm.get(), eps,
                                 _ctx.get(), R, sh, _stream));
  }

  // the mixer's output projection; what is left to add to the stream
  AddSpec project_out(const SudevikLayerWeight<T>& w, int k, int R, bool few) {
    const int W = _c.width;
    AddSpec add;
    add.row_stride = W;
    if (few) {
      int planes = 1;
      LSH_CALL(gemm_float_planes<T>(_ctx.get(), k, w.out.get(), _yf.get(), R, W, k, kMaxPlanes,
                                    &planes, _stream));
      add.y = _yf.get();
      add.parts = planes;
      add.part_stride = (long)R * W;
    } else {
      LSH_CALL((gemm_float<T, T>(_ctx.get(), k, w.out.get(), _y.get(), W, nullptr, 0, W, R, W, k,
                                 _stream)));
      add.y = _y.get();
      add.y_is_float = false;
      add.parts = 1;
    }
    return add;
  }

  // _h -> weighted expert outputs
  AddSpec experts(const SudevikLayerConfig& l, const SudevikLayerWeight<T>& w, int R, bool few) {
    const int W = _c.width;
    if (few) {
      LSH_CALL(moe_router<T>(_h.get(), w.router.get(), w.router_b.get(), _weight.get(), _count.get(),
                             _list.get(), R, W, l.experts, l.top, _stream));
    } else {
      LSH_CALL((gemm_float<T, float>(_h.get(), W, w.router.get(), _router.get(), l.experts, nullptr,
                                     0, l.experts, R, l.experts, W, _stream)));
      LSH_CALL(moe_route(_router.get(), w.router_b.get(), _weight.get(), _count.get(), _list.get(),
                         R, l.experts, l.top, _stream));
    }
    LSH_CALL(moe_up<T>(_h.get(), w.up.get(), _act.get(), _count.get(), _list.get(), R, l.top,
                       l.experts, W, l.ff, _stream));
    AddSpec add;
    add.parts = l.top;
    add.part_stride = W;
    add.row_stride = (long)l.top * W;
    add.weight = _weight.get();
    add.y_is_float = few;
    if (few) {
      LSH_CALL((moe_down<T, float>(_act.get(), w.down.get(), _exf.get(), _count.get(), _list.get(),
                                   R, l.top, l.experts, W, l.ff, _stream)));
      add.y = _exf.get();
    } else {
      LSH_CALL((moe_down<T, T>(_act.get(), w.down.get(), _ex.get(), _count.get(), _list.get(), R,
                               l.top, l.experts, W, l.ff, _stream)));
      add.y = _ex.get();
    }
    return add;
  }

  const SudevikConfig _c;
  const int _max_step, _slots;
  hipStream_t _stream;
  SudevikWeight<T> _w;
  std::vector<LayerCache<T>> _cache;
  std::vector<int> _rot;  // per layer: its table, or -1
  std::vector<std::pair<RotaryConfig, DeviceBuffer<float2>>> _tables;
  int _rows = 0, _seqs = 0, _wants = 0;
  DeviceBuffer<float> _x, _ba, _yf, _dq, _dk, _dg, _dbeta, _do, _chunk, _attn_ws, _router, _weight,
      _exf, _logits;
  DeviceBuffer<T> _h, _hf, _proj, _q, _ctx, _dv, _y, _act, _ex;
  DeviceBuffer<int> _count, _list;
};

}  // namespace

std::unique_ptr<DecoderStack> create_sudevik_stack(const SudevikConfig& config,
                                                   const SafeTensors& file, bool float32, int slots,
                                                   int max_step, hipStream_t stream) {
  if (float32) return std::make_unique<Stack<float>>(config, file, slots, max_step, stream);
  return std::make_unique<Stack<bf16_t>>(config, file, slots, max_step, stream);
}

}  // namespace hip
}  // namespace lightseq
