#include "decoder_lm.h"

#include <algorithm>

namespace lightseq {
namespace hip {

using namespace lsh;

DecoderLM::DecoderLM(const ModelOptions& options)
    : LSModel({"token_ids"}, {"result"}), _opt(options) {
  if (_opt.max_batch_size <= 0) throw std::runtime_error("max_batch_size must be positive");
  if (_opt.max_step <= 0) throw std::runtime_error("max_step must be positive");
  if (_opt.dtype != kBFloat16 && _opt.dtype != kFloat32)
    throw std::runtime_error("dtype must be bfloat16 or float32");
  if (_opt.topk < 0 || (_opt.topk == 0 && !(_opt.topp > 0.f && _opt.topp <= 1.f)))
    throw std::runtime_error("topk must be positive, or 0 with topp in (0, 1]");
}

void DecoderLM::open(const std::string& model_dir, int vocab, const BuildStack& build) {
  _vocab = vocab;
  CHECK_GPU_ERROR(hipSetDevice(0));
  stream_.create();
  {
    const SafeTensors file(model_dir + "/model.safetensors");
    _stack = build(file, _opt, stream_);
  }
  _slots = std::make_unique<SequenceSlots>(_opt.max_batch_size, _opt.max_step);
  const int B = _opt.max_batch_size;
  const size_t tokens = (size_t)B * _opt.max_step;
  d_input_.alloc(tokens);
  d_result_.alloc(tokens);
  _p_d_token_id = d_input_.get();
  _p_d_result = d_result_.get();
  _ids.alloc(tokens);
  for (DeviceBuffer<int>* b : {&_last_ids, &_row_slot, &_row_pos, &_row_len}) b->alloc(B);
  _unfinished.alloc(1);
  _rng.alloc(2 * (size_t)B);  // 16 bytes per row
  set_seed(0);
  CHECK_GPU_ERROR(hipHostMalloc(reinterpret_cast<void**>(&_h_unfinished), sizeof(int)));
  describe_input(0, kInt32, {B, _opt.max_step}, &_p_d_token_id);
  describe_output(0, kInt32, {B, _opt.max_step}, &_p_d_result);
  CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
}

DecoderLM::~DecoderLM() {
  if (stream_.get()) (void)hipStreamSynchronize(stream_);
  if (_h_batch) (void)hipHostFree(_h_batch);
  if (_h_unfinished) (void)hipHostFree(_h_unfinished);
}

void DecoderLM::set_seed(unsigned long long seed) {
  LSH_CALL(sample_state_setup(_rng.get(), _opt.max_batch_size, seed, stream_));
}

// Uploads a step's description and enqueues it; the previous step must have been synchronised.
const float* DecoderLM::enqueue(const std::vector<int>& slots, const std::vector<int>& counts,
                              const std::vector<int>& tokens, const std::vector<int>& want) {
  const int n = (int)slots.size();
  int rows = 0, max_n = 0, max_len = 0;
  for (int i = 0; i < n; ++i) {
    if (counts[i] <= 0) throw std::runtime_error("a step entry without tokens");
    for (int j = 0; j < i; ++j)
      if (slots[j] == slots[i]) throw std::runtime_error("a sequence appears twice in a step");
    const int len = _slots->length(slots[i]);
    if (len + counts[i] > _opt.max_step) throw std::runtime_error("sequence longer than max_step");
    rows += counts[i];
    max_n = std::max(max_n, counts[i]);
    max_len = std::max(max_len, len + counts[i]);
  }
  if ((int)tokens.size() != rows) throw std::runtime_error("token count mismatch");
  for (int t : tokens)
    if (t < 0 || t >= _vocab) throw std::runtime_error("token id outside the vocabulary");
  for (int r : want)
    if (r < 0 || r >= rows) throw std::runtime_error("wanted row outside the step");
  bool all = (int)want.size() == rows;
  for (int i = 0; all && i < rows; ++i) all = want[i] == i;

  const size_t ints = 3 * (size_t)rows + 4 * (size_t)n + want.size();
  if (ints > _batch_ints) {
    CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
    if (_h_batch) (void)hipHostFree(_h_batch);
    _h_batch = nullptr;
    _batch_ints = std::max(ints, 2 * _batch_ints);
    CHECK_GPU_ERROR(hipHostMalloc(reinterpret_cast<void**>(&_h_batch), _batch_ints * sizeof(int)));
    _batch.alloc(_batch_ints);
  }
  if (_stack->reserve(rows, n, (int)want.size())) _graphs.clear();
  int *ids = _h_batch, *slot = ids + rows, *pos = slot + rows, *span = pos + rows, *wp = span + 4 * n;
  static_assert(sizeof(SeqSpan) == 4 * sizeof(int), "a span is four ints");
  int r = 0;
  for (int i = 0; i < n; ++i) {
    const int len = _slots->length(slots[i]);
    const SeqSpan sp{r, counts[i], len, slots[i]};
    memcpy(span + 4 * i, &sp, sizeof(sp));
    for (int t = 0; t < counts[i]; ++t, ++r) {
      ids[r] = tokens[r];
      slot[r] = slots[i];
      pos[r] = len + t;
    }
  }
  std::copy(want.begin(), want.end(), wp);
  CHECK_GPU_ERROR(hipMemcpyAsync(_batch.get(), _h_batch, ints * sizeof(int), hipMemcpyHostToDevice,
                                 stream_));
  StepBatch b;
  b.rows = rows;
  b.n_seqs = n;
  b.max_n = max_n;
  b.max_len = max_len;
  b.ids = _batch.get();
  b.row_slot = b.ids + rows;
  b.row_pos = b.row_slot + rows;
  b.spans = reinterpret_cast<const SeqSpan*>(b.row_pos + rows);
  b.want = all ? nullptr : b.row_pos + rows + 4 * n;
  b.n_want = (int)want.size();
  const float* logits = _stack->run(b, _taps, _steps_run);
  for (int i = 0; i < n; ++i) _slots->advance(slots[i], counts[i]);
  return logits;
}

void DecoderLM::step(const std::vector<int>& slots, const std::vector<int>& counts,
                   const std::vector<int>& tokens, const std::vector<int>& want,
                   float* host_logits) {
  const float* logits = enqueue(slots, counts, tokens, want);
  ++_steps_run;
  if (!want.empty())
    CHECK_GPU_ERROR(hipMemcpyAsync(host_logits, logits,
                                   want.size() * (size_t)_vocab * sizeof(float),
                                   hipMemcpyDeviceToHost, stream_));
  CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
}

void DecoderLM::sample(const float* logits, int batch) {
  LSH_CALL(lm_sample(logits, batch, _vocab, _opt.topk, _opt.topp,
                     _is_benchmark ? -1 : _opt.eos_id, _rng.get(), _ids.get(), _opt.max_step,
                     _last_ids.get(), _row_len.get(), _row_pos.get(), _unfinished.get(), stream_));
}

// Prompts of `lengths` tokens in `tokens`; leaves the texts in _ids and their lengths in `lengths`.
int DecoderLM::generate(const std::vector<int>& slots, std::vector<int>& lengths,
                      const std::vector<int>& tokens) {
  const int B = (int)slots.size(), S = _opt.max_step;
  const int longest = *std::max_element(lengths.begin(), lengths.end());
  const int limit = std::min(S, longest + std::max(_opt.extra_decode_length, 0));
  _steps_run = 0;
  _phases.mark(0, stream_);
  LSH_CALL(fill_i32(_ids.get(), _opt.padding_id, B * S, stream_));
  LSH_CALL(fill_i32(_unfinished.get(), 0, 1, stream_));
  int at = 0;
  std::vector<int> want;
  for (int i = 0; i < B; ++i) {
    CHECK_GPU_ERROR(hipMemcpyAsync(_ids.get() + (size_t)i * S, tokens.data() + at,
                                   sizeof(int) * lengths[i], hipMemcpyHostToDevice, stream_));
    at += lengths[i];
    want.push_back(at - 1);
  }
  _row_slot.upload(slots.data(), B, stream_);
  _row_len.upload(lengths.data(), B, stream_);
  // room for the decoding steps too, so that nothing moves between them
  _stack->reserve((int)tokens.size(), B, B);
  const float* logits = enqueue(slots, lengths, tokens, want);
  int loop_steps = 0;
  const auto unfinished = [&] {
    if (_is_benchmark) return 1;  // nothing stops a benchmark run but the length
    CHECK_GPU_ERROR(hipMemcpyAsync(_h_unfinished, _unfinished.get(), sizeof(int),
                                   hipMemcpyDeviceToHost, stream_));
    CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
    return *_h_unfinished;
  };
  int len = longest;  // of the longest row, counting ended rows as if they went on
  if (len < limit) {
    sample(logits, B);
    ++len;
    ++_steps_run;
    int go_on = unfinished();
    _phases.mark(1, stream_);
    StepBatch b;
    b.rows = b.n_seqs = b.n_want = B;
    b.max_n = 1;
    b.ids = _last_ids.get();
    b.row_slot = _row_slot.get();
    b.row_pos = _row_pos.get();
    b.zero_flag = _unfinished.get();
    while (go_on && len < limit) {
      // the launches of a step depend on the batch size and on this bound only
      b.max_len = std::min(S, (len + 255) / 256 * 256);
      const uint64_t key = ((uint64_t)B << 40) | ((uint64_t)b.max_len << 1) | (_is_benchmark ? 1 : 0);
      _graphs.run(key, stream_, _use_graphs && !_taps.any(),
                  [&] { sample(_stack->run(b, _taps, _steps_run), B); });
      ++loop_steps;
      ++len;
      ++_steps_run;
      go_on = unfinished();
    }
  } else {
    _phases.mark(1, stream_);
  }
  _phases.mark(2, stream_);
  _phases.set_loop_steps(loop_steps);
  CHECK_GPU_ERROR(hipMemcpyAsync(lengths.data(), _row_len.get(), sizeof(int) * B,
                                 hipMemcpyDeviceToHost, stream_));
  CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
  int out = 0;
  for (int& n : lengths) {
    if (n < 0) n = -n;  // ended
    out = std::max(out, n);
  }
  return out;
}

void DecoderLM::Infer() {
  if (input_shapes_[0].size() != 2) throw std::runtime_error("token_ids must be 2-D");
  const int B = input_shapes_[0][0], L = input_shapes_[0][1];
  if (B > _opt.max_batch_size)
    throw std::runtime_error("batch size of input greater than max_batch_size");
  if (L > _opt.max_step) throw std::runtime_error("seq len of input greater than max_step");
  if (B <= 0 || L <= 0) throw std::runtime_error("empty input");
  std::vector<int> in((size_t)B * L), lengths(B), tokens, slots;
  CHECK_GPU_ERROR(hipMemcpyAsync(in.data(), _p_d_token_id, in.size() * sizeof(int),
                                 hipMemcpyDeviceToHost, stream_));
  CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
  for (int i = 0; i < B; ++i) {
    int n = L;
    while (n > 0 && in[(size_t)i * L + n - 1] == _opt.padding_id) --n;
    if (n == 0) throw std::runtime_error("a prompt without tokens");
    lengths[i] = n;
    tokens.insert(tokens.end(), in.begin() + (size_t)i * L, in.begin() + (size_t)i * L + n);
  }
  struct Closer {
    SequenceSlots* s;
    std::vector<int>& open;
    ~Closer() {
      for (int x : open) s->close(x);
    }
  } closer{_slots.get(), slots};
  for (int i = 0; i < B; ++i) slots.push_back(_slots->open());
  const int out = generate(slots, lengths, tokens);
  CHECK_GPU_ERROR(hipMemcpy2DAsync(_p_d_result, sizeof(int) * out, _ids.get(),
                                   sizeof(int) * _opt.max_step, sizeof(int) * out, B,
                                   hipMemcpyDeviceToDevice, stream_));
  CHECK_GPU_ERROR(hipStreamSynchronize(stream_));
  set_output_shape(0, {B, out});
}

}  // namespace hip
}  // namespace lightseq
