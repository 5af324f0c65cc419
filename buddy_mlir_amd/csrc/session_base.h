// session_base.h -- what every resident decoder session has, whatever model it
// runs: the stream, the step state on the device (token, position, step count), the
// log of greedy tokens, the captured decode steps, the logits.  A model class
// supplies its layers; the exported session calls (session.hip) work on this.
#pragma once

#include "common.h"

#include <map>
#include <utility>
#include <vector>

namespace bh {

struct Qwen2Session;

struct Session {
  virtual ~Session();

  // ---- the model's part
  virtual const char *architecture() const = 0;
  // weights complete?
  virtual int ready() const = 0;
  // The next token will stand at `pos`: refuses positions the model's state cannot
  // continue from; position 0 begins a new sequence.
  virtual int seek(int pos) = 0;
  // Enqueues one decode step for the token and position in device memory; `pos` is
  // the host's copy of the position.  Steps with equal keys enqueue equal work.
  virtual std::pair<int, int> step_key(int pos) const = 0;
  virtual int enqueue_step(int pos) = 0;
  virtual void stepped() {}
  // what a step finds prepared once the host has written token and position
  virtual int prepare_step() = 0;
  // Runs n tokens (host or device) from `start` on and leaves the logits of the
  // asked-for rows (ascending, host) in dst ([n_rows][vocab], device).
  virtual int prefill_rows(const int *tokens, int n, int start, const int *rows, int n_rows,
                           float *dst) = 0;
  // forgets the sequence
  virtual int reset() = 0;
  // rows of a [kv_heads, max_len, head_dim] cache, for callers that mirror it
  virtual int copy_kv_rows(int, int, float *) {
    return fail(BUDDY_HIP_ERR_ARG, "%s keeps no cache of per-head keys and values", architecture());
  }
  virtual Qwen2Session *qwen2() { return nullptr; }

  // ---- shared
  hipStream_t stream = nullptr;
  bool own_stream = false;
  int vocab = 0, max_len = 0;
  float *logits = nullptr;
  void *amax_ws = nullptr;
  float *group_max_v = nullptr; // first maxima of the head's channel groups: values,
  int *group_max_i = nullptr;   // indices
  int *state = nullptr;         // device: token, pos, step
  int *token_log = nullptr;     // device: greedy tokens by step
  int token_log_cap = 0;
  int *host_state = nullptr;    // pinned staging for token/pos/step
  // Host-side mirror of the device's (position, step): what the next enqueued
  // step will use.  -1 until set_state; every step advances both on the device,
  // so the host can refuse steps that would leave the cache or the token log.
  int next_pos = -1, next_step = 0;
  struct StepGraph {
    hipGraph_t graph = nullptr;
    hipGraphExec_t exec = nullptr;
  };
  std::map<std::pair<int, int>, StepGraph> graphs; // one captured step per key
  static constexpr size_t kMaxStepGraphs = 8;
  bool use_graph = true;
  std::vector<void *> owned;

  template <typename T> int alloc(T **p, size_t n) {
    void *q = nullptr;
    BH_CHECK_HIP(hipMalloc(&q, n * sizeof(T)));
    owned.push_back(q);
    *p = static_cast<T *>(q);
    return BUDDY_HIP_OK;
  }
  // stream (null: one of its own) and the buffers above
  int init(int vocab_size, int capacity, hipStream_t on_stream);
  void drop_graph();
  int invalidate_graph();
  int check_steps(int steps, const char *who) const;
  int run_step();
  int set_state(int token, int pos, int step);
};

inline Session *as_session(buddy_hip_session *s) { return reinterpret_cast<Session *>(s); }
inline buddy_hip_session *as_handle(Session *s) { return reinterpret_cast<buddy_hip_session *>(s); }

} // namespace bh
