// trace_run -- replays given token ids through a model folder, step by step, and
// writes the logits that are asked for.  Nothing is sampled: a portion of a prompt
// goes through the session's prefill, a single token through its decode step, the
// same calls that generation makes.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]
//
// Steps come on standard input, one JSON object a line:
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
// `want`: places among these tokens whose logits are written; `end`: sequences that
// are finished.  DIR/<step>.f32 receives [wanted, vocab] little-endian floats, and
// "done <step>" is printed after every step.  One sequence is live at a time.
#include <algorithm>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <exception>
#include <iostream>
#include <string>
#include <vector>

#include "buddy_hip/buddy_hip.h"
#include "json.h"

namespace {

int usage() {
  fputs("usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]\n", stderr);
  return 2;
}

int failed(const std::string &what) {
  fprintf(stderr, "[Error] %s\n", what.c_str());
  return 1;
}

struct Replay {
  buddy_hip_session *session = nullptr;
  int vocab = 0;
  std::string live; // the sequence the session holds
  bool any = false;
  int position = 0;

  // The logits of `want`, appended in its order.
  int portion(const std::vector<int> &tokens, const std::vector<int> &want, std::vector<float> &out) {
    std::vector<int> rows = want;
    std::sort(rows.begin(), rows.end());
    rows.erase(std::unique(rows.begin(), rows.end()), rows.end());
    for (int r : rows)
      if (r < 0 || r >= (int)tokens.size())
        return failed("a wanted place lies outside the tokens");
    for (int t : tokens)
      if (t < 0 || t >= vocab)
        return failed("token id outside the vocabulary");
    std::vector<float> logits(std::max<size_t>(rows.size(), 1) * (size_t)vocab);
    int rc;
    if (tokens.size() == 1)
      rc = buddy_hip_session_decode(session, tokens[0], position, logits.data(), nullptr);
    else
      rc = buddy_hip_session_prefill_rows(session, tokens.data(), (int)tokens.size(), position,
                                          rows.data(), (int)rows.size(), logits.data());
    if (rc)
      return failed(buddy_hip_last_error());
    position += (int)tokens.size();
    for (int w : want) {
      const size_t r = (size_t)(std::lower_bound(rows.begin(), rows.end(), w) - rows.begin());
      out.insert(out.end(), logits.begin() + (long)(r * vocab), logits.begin() + (long)((r + 1) * vocab));
    }
    return 0;
  }
};

std::vector<int> integers(const bh::Json &j) {
  std::vector<int> v;
  for (const bh::Json &e : j.array())
    v.push_back((int)e.integer());
  return v;
}

int replay(Replay &r, const std::string &out_dir) {
  std::string line;
  while (std::getline(std::cin, line)) {
    if (line.find_first_not_of(" \t\r") == std::string::npos)
      continue;
    const bh::Json j = bh::Json::parse(line);
    const long long step = j.at("step").integer();
    std::vector<float> out;
    for (const bh::Json &e : j.at("entries").array()) {
      const std::string &id = e.at("id").string();
      const std::vector<int> tokens = integers(e.at("tokens"));
      if (tokens.empty())
        continue;
      if (!r.any) {
        if (buddy_hip_session_reset(r.session))
          return failed(buddy_hip_last_error());
        r.any = true;
        r.live = id;
        r.position = 0;
      } else if (r.live != id) {
        return failed("sequence " + id + " begins before " + r.live + " has ended");
      }
      const bh::Json *want = e.find("want");
      if (int rc = r.portion(tokens, want ? integers(*want) : std::vector<int>(), out))
        return rc;
    }
    if (const bh::Json *end = j.find("end"))
      for (const bh::Json &id : end->array())
        if (r.any && id.string() == r.live) {
          if (buddy_hip_session_reset(r.session))
            return failed(buddy_hip_last_error());
          r.any = false;
        }
    if (!out.empty()) {
      const std::string path = out_dir + "/" + std::to_string(step) + ".f32";
      FILE *f = fopen(path.c_str(), "wb");
      const bool ok = f && fwrite(out.data(), sizeof(float), out.size(), f) == out.size();
      if ((f && fclose(f)) || !ok)
        return failed("cannot write " + path);
    }
    printf("done %lld\n", step);
    fflush(stdout);
  }
  return 0;
}

} // namespace

int main(int argc, char **argv) {
  std::string model, dtype, out;
  long max_tokens = 0;
  for (int i = 1; i + 1 < argc; i += 2) {
    const std::string a = argv[i];
    if (a == "--model") model = argv[i + 1];
    else if (a == "--dtype") dtype = argv[i + 1];
    else if (a == "--out") out = argv[i + 1];
    else if (a == "--max-tokens") max_tokens = atol(argv[i + 1]);
    else return usage();
  }
  if (argc % 2 == 0 || model.empty() || out.empty() || max_tokens < 0 || max_tokens > (1 << 24) ||
      (dtype != "bfloat16" && dtype != "float32"))
    return usage();
  buddy_hip_model_options o = {};
  o.dtype = dtype == "float32" ? BUDDY_HIP_MODEL_F32 : BUDDY_HIP_MODEL_BF16;
  o.max_len = max_tokens ? (int)max_tokens : 65536;
  Replay r;
  r.session = buddy_hip_session_create_from_folder(model.c_str(), &o);
  if (!r.session)
    return failed(buddy_hip_last_error());
  r.vocab = buddy_hip_session_vocab(r.session);
  int rc;
  try {
    rc = replay(r, out);
  } catch (const std::exception &e) {
    rc = failed(e.what());
  }
  buddy_hip_session_destroy(r.session);
  return rc;
}
