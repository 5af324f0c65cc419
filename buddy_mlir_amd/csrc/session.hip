// session.hip -- resident decoder sessions: the exported calls that do not depend on
// the model, and the part of a session every model shares.
//
// Takes the place of the generated ModelSession
// (tools/buddy-codegen/gen_session.py:1381-1452) and of the greedy part of the
// decode loop (runtime/llm/TextGeneration.cpp:215-266, Sampler.h:101-104).  Token
// id, position and step counter live in device memory, so a whole decode step is
// captured once into a hipGraph and replayed; greedy decoding feeds the argmax
// straight into the next step's embedding gather without a host round trip.
#include "session_base.h"
#include "elementwise.h"

#include <vector>

namespace bh {

Session::~Session() {
  if (stream)
    (void)hipStreamSynchronize(stream);
  drop_graph();
  for (void *p : owned)
    (void)hipFree(p);
  if (host_state)
    (void)hipHostFree(host_state);
  if (own_stream)
    (void)hipStreamDestroy(stream);
}

int Session::init(int vocab_size, int capacity, hipStream_t on_stream) {
  vocab = vocab_size;
  max_len = capacity;
  stream = on_stream;
  if (!stream) {
    BH_CHECK_HIP(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
    own_stream = true;
  }
  const size_t groups = (size_t)ceil_div(vocab, kTileN);
  token_log_cap = 65536;
  int rc = alloc(&logits, groups * kTileN);
  rc |= alloc(&state, 4);
  rc |= alloc(&token_log, (size_t)token_log_cap);
  rc |= alloc((char **)&amax_ws, argmax_workspace_bytes());
  rc |= alloc(&group_max_v, groups);
  rc |= alloc(&group_max_i, groups);
  if (rc)
    return rc;
  BH_CHECK_HIP(hipHostMalloc((void **)&host_state, 4 * sizeof(int)));
  BH_CHECK_HIP(hipMemsetAsync(state, 0, 4 * sizeof(int), stream));
  BH_CHECK_HIP(hipStreamSynchronize(stream));
  return BUDDY_HIP_OK;
}

void Session::drop_graph() {
  for (auto &kv : graphs) {
    if (kv.second.exec)
      (void)hipGraphExecDestroy(kv.second.exec);
    if (kv.second.graph)
      (void)hipGraphDestroy(kv.second.graph);
  }
  graphs.clear();
}

// The position and step the device holds must stay inside the cache and the
// token log for every one of `steps` further steps.
int Session::check_steps(int steps, const char *who) const {
  BH_REQUIRE(next_pos >= 0, "%s: no token / position set (set_state first)", who);
  BH_REQUIRE(steps > 0 && (int64_t)next_pos + steps <= max_len,
             "%s: %d step(s) from position %d leave the cache (max_len %d)", who, steps,
             next_pos, max_len);
  BH_REQUIRE((int64_t)next_step + steps <= token_log_cap,
             "%s: %d step(s) from step %d overflow the token log (%d entries)", who,
             steps, next_step, token_log_cap);
  return BUDDY_HIP_OK;
}

int Session::run_step() {
  int rc = check_steps(1, "decode step");
  if (rc)
    return rc;
  if (!use_graph) {
    rc = enqueue_step(next_pos);
  } else {
    const std::pair<int, int> key = step_key(next_pos);
    auto it = graphs.find(key);
    if (it == graphs.end()) {
      if (graphs.size() >= kMaxStepGraphs) {
        BH_CHECK_HIP(hipStreamSynchronize(stream)); // a replay may still be running
        drop_graph();
      }
      it = graphs.emplace(key, StepGraph{}).first;
    }
    StepGraph &g = it->second;
    if (!g.exec) {
      BH_CHECK_HIP(hipStreamBeginCapture(stream, hipStreamCaptureModeThreadLocal));
      rc = enqueue_step(next_pos);
      hipError_t e = hipStreamEndCapture(stream, &g.graph);
      if (!rc && e != hipSuccess)
        rc = fail(BUDDY_HIP_ERR_HIP, "hipStreamEndCapture: %s", hipGetErrorString(e));
      if (!rc && (e = hipGraphInstantiate(&g.exec, g.graph, nullptr, nullptr, 0)) != hipSuccess)
        rc = fail(BUDDY_HIP_ERR_HIP, "hipGraphInstantiate: %s", hipGetErrorString(e));
      if (rc) {
        drop_graph(); // a half-built graph is not kept
        return rc;
      }
    }
    BH_CHECK_HIP(hipGraphLaunch(g.exec, stream));
  }
  if (!rc) {
    ++next_pos;
    ++next_step;
    stepped();
  }
  return rc;
}

// The captured step has kernel arguments baked in (weight, cache and embedding
// pointers): whoever may change one of them drops the graph first, and the
// next step captures a new one.
int Session::invalidate_graph() {
  if (!graphs.empty()) {
    BH_CHECK_HIP(hipStreamSynchronize(stream));
    drop_graph();
  }
  return BUDDY_HIP_OK;
}

int Session::set_state(int token, int pos, int step) {
  int rc = seek(pos);
  if (rc)
    return rc;
  next_pos = pos;
  next_step = step;
  host_state[0] = token;
  host_state[1] = pos;
  host_state[2] = step;
  BH_CHECK_HIP(hipMemcpyAsync(state, host_state, 3 * sizeof(int),
                              hipMemcpyHostToDevice, stream));
  if ((rc = prepare_step()))
    return rc;
  // the pinned staging words are reused by the next call
  BH_CHECK_HIP(hipStreamSynchronize(stream));
  return BUDDY_HIP_OK;
}

} // namespace bh

using bh::Session;

extern "C" {

void buddy_hip_session_destroy(buddy_hip_session *hs) try {
  delete bh::as_session(hs);
} BH_CATCH_VOID("buddy_hip_session_destroy")

int buddy_hip_session_use_graph(buddy_hip_session *hs, int enable) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s, "session_use_graph: null session");
  s->use_graph = enable != 0;
  return BUDDY_HIP_OK;
} BH_CATCH_INT("buddy_hip_session_use_graph")

int buddy_hip_session_decode_mirror(buddy_hip_session *hs, int token, int pos,
                                    float *logits_out, float *kv_rows_out,
                                    int *next_token) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s, "session_decode: null session");
  int rc = s->ready();
  if (rc)
    return rc;
  BH_REQUIRE(token >= 0 && token < s->vocab, "session_decode: token %d", token);
  BH_REQUIRE(pos >= 0 && pos < s->max_len,
             "session_decode: position %d outside the cache (max_len %d)", pos,
             s->max_len);
  if ((rc = s->set_state(token, pos, 0)))
    return rc;
  if ((rc = s->run_step()))
    return rc;
  if (logits_out)
    BH_CHECK_HIP(hipMemcpyAsync(logits_out, s->logits,
                                sizeof(float) * s->vocab, hipMemcpyDefault,
                                s->stream));
  BH_CHECK_HIP(hipMemcpyAsync(s->host_state, s->state, 3 * sizeof(int),
                              hipMemcpyDeviceToHost, s->stream));
  if (kv_rows_out) { // the cache rows this step wrote, all layers
    if ((rc = s->copy_kv_rows(pos, 1, kv_rows_out)))
      return rc;
  }
  BH_CHECK_HIP(hipStreamSynchronize(s->stream));
  if (next_token)
    *next_token = s->host_state[0];
  return BUDDY_HIP_OK;
} BH_CATCH_INT("buddy_hip_session_decode_mirror")

int buddy_hip_session_decode(buddy_hip_session *hs, int token, int pos,
                             float *logits_out, int *next_token) {
  return buddy_hip_session_decode_mirror(hs, token, pos, logits_out, nullptr, next_token);
}

int buddy_hip_session_decode_greedy(buddy_hip_session *hs, int first_token,
                                    int start_pos, int steps, int *tokens_out) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s && tokens_out, "session_decode_greedy: null argument");
  int rc = s->ready();
  if (rc)
    return rc;
  BH_REQUIRE(first_token >= 0 && first_token < s->vocab,
             "session_decode_greedy: token %d", first_token);
  BH_REQUIRE(steps > 0 && steps <= s->token_log_cap,
             "session_decode_greedy: steps %d", steps);
  BH_REQUIRE(start_pos >= 0 && start_pos + steps <= s->max_len,
             "session_decode_greedy: positions %d..%d outside the cache (max_len %d)",
             start_pos, start_pos + steps - 1, s->max_len);
  if ((rc = s->set_state(first_token, start_pos, 0)))
    return rc;
  for (int i = 0; i < steps; ++i)
    if ((rc = s->run_step()))
      return rc;
  BH_CHECK_HIP(hipMemcpyAsync(tokens_out, s->token_log, sizeof(int) * steps,
                              hipMemcpyDefault, s->stream));
  BH_CHECK_HIP(hipStreamSynchronize(s->stream));
  return BUDDY_HIP_OK;
} BH_CATCH_INT("buddy_hip_session_decode_greedy")

int buddy_hip_session_prefill(buddy_hip_session *hs, const int *tokens,
                              int n_tokens, int start_pos, float *logits_out,
                              int *next_token) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s && tokens, "session_prefill: null argument");
  int rc = s->ready();
  if (rc)
    return rc;
  BH_REQUIRE(n_tokens > 0 && start_pos >= 0 && start_pos + n_tokens <= s->max_len,
             "session_prefill: tokens %d..%d outside the cache (max_len %d)",
             start_pos, start_pos + n_tokens - 1, s->max_len);
  const int last = n_tokens - 1;
  if ((rc = s->prefill_rows(tokens, n_tokens, start_pos, &last, 1, s->logits)))
    return rc;
  if ((rc = bh::launch_argmax(s->logits, s->vocab, s->amax_ws, s->state, nullptr,
                              nullptr, s->stream)))
    return rc;
  if (logits_out)
    BH_CHECK_HIP(hipMemcpyAsync(logits_out, s->logits, sizeof(float) * s->vocab,
                                hipMemcpyDefault, s->stream));
  BH_CHECK_HIP(hipMemcpyAsync(s->host_state, s->state, sizeof(int),
                              hipMemcpyDeviceToHost, s->stream));
  BH_CHECK_HIP(hipStreamSynchronize(s->stream));
  if (next_token)
    *next_token = s->host_state[0];
  return BUDDY_HIP_OK;
} BH_CATCH_INT("buddy_hip_session_prefill")

int buddy_hip_session_prefill_rows(buddy_hip_session *hs, const int *tokens, int n_tokens,
                                   int start_pos, const int *rows, int n_rows,
                                   float *logits_out) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s && tokens && n_rows >= 0 && (n_rows == 0 || (rows && logits_out)),
             "session_prefill_rows: null argument");
  int rc = s->ready();
  if (rc)
    return rc;
  BH_REQUIRE(n_tokens > 0 && start_pos >= 0 && (int64_t)start_pos + n_tokens <= s->max_len,
             "session_prefill_rows: tokens %d..%d outside the cache (max_len %d)", start_pos,
             start_pos + n_tokens - 1, s->max_len);
  for (int i = 0; i < n_rows; ++i)
    BH_REQUIRE(rows[i] >= 0 && rows[i] < n_tokens && (i == 0 || rows[i] > rows[i - 1]),
               "session_prefill_rows: rows must ascend within the tokens");
  float *dev = nullptr;
  const size_t bytes = sizeof(float) * (size_t)n_rows * s->vocab;
  if (n_rows)
    BH_CHECK_HIP(hipMalloc((void **)&dev, bytes));
  rc = s->prefill_rows(tokens, n_tokens, start_pos, rows, n_rows, dev);
  if (!rc && n_rows &&
      hipMemcpyAsync(logits_out, dev, bytes, hipMemcpyDefault, s->stream) != hipSuccess)
    rc = bh::fail(BUDDY_HIP_ERR_HIP, "session_prefill_rows: copy failed");
  const hipError_t e = hipStreamSynchronize(s->stream);
  if (!rc && e != hipSuccess)
    rc = bh::fail(BUDDY_HIP_ERR_HIP, "session_prefill_rows: %s", hipGetErrorString(e));
  if (dev)
    (void)hipFree(dev);
  return rc;
} BH_CATCH_INT("buddy_hip_session_prefill_rows")

int buddy_hip_session_prefill_all_logits(buddy_hip_session *hs, const int *tokens,
                                         int n_tokens, int start_pos,
                                         float *logits_out) try {
  BH_REQUIRE(hs && tokens && logits_out && n_tokens > 0,
             "session_prefill_all_logits: bad argument");
  std::vector<int> rows((size_t)n_tokens);
  for (int i = 0; i < n_tokens; ++i)
    rows[(size_t)i] = i;
  return buddy_hip_session_prefill_rows(hs, tokens, n_tokens, start_pos, rows.data(), n_tokens,
                                        logits_out);
} BH_CATCH_INT("buddy_hip_session_prefill_all_logits")

void buddy_hip_session_adopt(buddy_hip_session *hs, void *device_ptr) try {
  Session *s = bh::as_session(hs);
  if (s && device_ptr)
    s->owned.push_back(device_ptr);
} BH_CATCH_VOID("buddy_hip_session_adopt")

int buddy_hip_session_enqueue_steps(buddy_hip_session *hs, int steps) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s && steps > 0, "session_enqueue_steps: bad argument");
  int rc = s->ready();
  if (rc)
    return rc;
  // refused as a whole: no step is enqueued when the last one would not fit
  if ((rc = s->check_steps(steps, "session_enqueue_steps")))
    return rc;
  for (int i = 0; i < steps; ++i)
    if ((rc = s->run_step()))
      return rc;
  return BUDDY_HIP_OK;
} BH_CATCH_INT("buddy_hip_session_enqueue_steps")

int buddy_hip_session_set_state(buddy_hip_session *hs, int token, int pos) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s, "session_set_state: null session");
  BH_REQUIRE(token >= 0 && token < s->vocab && pos >= 0 &&
                 pos < s->max_len,
             "session_set_state: token %d / position %d out of range", token, pos);
  int rc = s->ready();
  if (rc)
    return rc;
  return s->set_state(token, pos, 0);
} BH_CATCH_INT("buddy_hip_session_set_state")

const float *buddy_hip_session_logits(buddy_hip_session *hs) {
  Session *s = bh::as_session(hs);
  return s ? s->logits : nullptr;
}

int buddy_hip_session_reset(buddy_hip_session *hs) try {
  Session *s = bh::as_session(hs);
  BH_REQUIRE(s, "session_reset: null session");
  s->next_pos = -1; // the next step needs a token and a position first
  return s->reset();
} BH_CATCH_INT("buddy_hip_session_reset")

const char *buddy_hip_session_architecture(buddy_hip_session *hs) {
  return hs ? bh::as_session(hs)->architecture() : nullptr;
}

int buddy_hip_session_vocab(buddy_hip_session *hs) try {
  Session *s = bh::as_session(hs);
  return s ? s->vocab : 0;
} BH_CATCH_INT("buddy_hip_session_vocab")

buddy_hip_stream buddy_hip_session_stream(buddy_hip_session *hs) {
  Session *s = bh::as_session(hs);
  return s ? reinterpret_cast<buddy_hip_stream>(s->stream) : nullptr;
}
}
