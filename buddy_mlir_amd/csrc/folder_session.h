// folder_session.h -- what the model classes built from a folder share: weights onto
// the device as bfloat16 tiles, one sequence that continues where its state stands, a
// prompt in blocks, the head's rows of logits.
#pragma once

#include "bf16_linear.h"
#include "model_registry.h"
#include "row_ops.h"

#include <algorithm>
#include <new>
#include <stdexcept>
#include <string>
#include <vector>

namespace bh {

// a size of a configuration
inline int positive(const Json &j, const char *key) {
  const int64_t v = j.at(key).integer();
  if (v <= 0 || v > (1 << 24))
    throw std::runtime_error(std::string("config: \"") + key + "\" out of range");
  return (int)v;
}

// One input of a fused projection: where its channels lie in the result.
struct Part {
  int at = 0, n = 0;
};

inline int pow2_at_least(int64_t v) {
  int p = 2;
  while (p < v)
    p *= 2;
  return p;
}

struct FolderSession : Session {
  ModelOptions opt;
  int seq_len = 0; // tokens the state holds

  // a block of a prompt, grown on demand to `pf_rows` rows
  int pf_rows = 0;
  std::vector<void *> pf_owned;
  int *pf_tokens = nullptr, *pf_pick = nullptr;
  static constexpr int kLogitRows = 256; // rows of the head multiplied at once

  explicit FolderSession(const ModelOptions &o) : opt(o) {}
  ~FolderSession() override {
    if (stream)
      (void)hipStreamSynchronize(stream);
    free_block();
  }

  // ---- the model's part
  // (re)allocates what a block of `rows` tokens needs, with block_alloc
  virtual int alloc_block(int rows) = 0;
  // One block of tokens (in pf_tokens) through all layers; the logits of the rows
  // listed (host, ascending) go to dst.
  virtual int run_block(int n, int start, const int *rows, int n_rows, float *dst) = 0;

  // ---- loading
  // a bfloat16 tensor on the device, freed when it goes out of scope
  struct Upload {
    uint16_t *p = nullptr;
    Upload(const TensorView &t, hipStream_t stream) {
      if (hipMalloc((void **)&p, t.bytes) != hipSuccess)
        throw std::bad_alloc();
      if (hipMemcpyAsync(p, t.data, t.bytes, hipMemcpyHostToDevice, stream) != hipSuccess) {
        (void)hipFree(p);
        throw std::runtime_error("upload failed");
      }
    }
    ~Upload() { (void)hipFree(p); } // waits for the work that reads it
    Upload(const Upload &) = delete;
    Upload &operator=(const Upload &) = delete;
  };
  void must(int rc) {
    if (rc)
      throw std::runtime_error(buddy_hip_last_error());
  }
  template <typename T> T *device(size_t n) {
    T *p = nullptr;
    must(alloc(&p, n));
    return p;
  }
  template <typename T> T *device_copy(const std::vector<T> &v) {
    T *p = device<T>(v.size());
    if (hipMemcpy(p, v.data(), v.size() * sizeof(T), hipMemcpyHostToDevice) != hipSuccess)
      throw std::runtime_error("upload failed");
    return p;
  }
  template <typename T> T *device_zeros(size_t n) {
    T *p = device<T>(n);
    if (hipMemsetAsync(p, 0, n * sizeof(T), stream) != hipSuccess)
      throw std::runtime_error("clear failed");
    return p;
  }
  uint16_t *device_bf16(const TensorView &t) {
    uint16_t *p = device<uint16_t>((size_t)t.count());
    if (hipMemcpy(p, t.data, t.bytes, hipMemcpyHostToDevice) != hipSuccess)
      throw std::runtime_error("upload failed");
    return p;
  }
  Bf16Matrix matrix(int64_t N, int64_t K) {
    Bf16Matrix m;
    m.N = (int)round_up(N, 16);
    m.K = (int)K;
    m.ktiles = bf16_ktiles(K);
    m.tiles = reinterpret_cast<const uint4 *>(device<char>(bf16_tiles_bytes(K, N)));
    return m;
  }
  // packs `src` (element (n, k) at n * sn + k * sk) as channels from `at` on
  void pack(const Bf16Matrix &m, int at, const uint16_t *src, int64_t sn, int64_t sk, int64_t N) {
    must(launch_pack_bf16(src, sn, sk, N, m.K,
                          const_cast<uint4 *>(m.tiles) + (int64_t)(at / 16) * m.ktiles * 64, stream));
  }
  Bf16Matrix load_matrix(const ModelFolder &f, const std::string &name, int64_t N, int64_t K) {
    Upload u(f.bf16(name, {N, K}), stream);
    Bf16Matrix m = matrix(N, K);
    pack(m, 0, u.p, K, 1, N);
    return m;
  }
  // Several matrices on the same input as one, each from a multiple of 16 channels on.
  Bf16Matrix load_parts(const ModelFolder &f, const std::string &prefix,
                        const std::vector<std::pair<std::string, Part *>> &parts, int64_t K) {
    int at = 0;
    for (auto &part : parts) {
      part.second->at = at;
      at += (int)round_up(part.second->n, 16);
    }
    const Bf16Matrix m = matrix(at, K);
    for (auto &part : parts) {
      Upload u(f.bf16(prefix + part.first, {part.second->n, K}), stream);
      pack(m, part.second->at, u.p, K, 1, part.second->n);
    }
    return m;
  }

  // ---- the sequence
  int ready() const override { return BUDDY_HIP_OK; }
  int seek(int pos) override {
    if (pos == 0)
      return seq_len == 0 ? BUDDY_HIP_OK : reset();
    BH_REQUIRE(pos == seq_len,
               "%s: position %d asked for, but the state holds %d tokens (continue there, or "
               "begin at 0)",
               architecture(), pos, seq_len);
    return BUDDY_HIP_OK;
  }
  void stepped() override { ++seq_len; }
  // Keys the attention launches of a step cover: the number of visible ones rounded up
  // to a quarter of a power of two, so that a few captured steps serve all positions.
  static int key_span(int visible) {
    int unit = 64;
    while (unit * 8 <= visible)
      unit *= 2;
    return (int)round_up(visible, unit);
  }

  // ---- many tokens
  void free_block() {
    for (void *p : pf_owned)
      (void)hipFree(p);
    pf_owned.clear();
    pf_rows = 0;
  }
  template <typename T> int block_alloc(T **p, size_t bytes) {
    void *q = nullptr;
    BH_CHECK_HIP(hipMalloc(&q, std::max<size_t>(bytes, 16)));
    pf_owned.push_back(q);
    *p = static_cast<T *>(q);
    return BUDDY_HIP_OK;
  }
  int ensure_block(int rows) {
    if (rows <= pf_rows)
      return BUDDY_HIP_OK;
    BH_CHECK_HIP(hipStreamSynchronize(stream));
    free_block();
    int rc = block_alloc(&pf_tokens, 4 * (size_t)rows);
    rc |= block_alloc(&pf_pick, 4 * (size_t)rows);
    rc |= alloc_block(rows);
    if (rc)
      return rc;
    pf_rows = rows;
    return BUDDY_HIP_OK;
  }
  RowsGemm gemm(const Bf16Matrix &W, const void *A, int lda, int rows, GemmOut out, void *C,
                int ldc) const {
    RowsGemm g;
    g.W = W;
    g.A = A;
    g.lda = lda;
    g.f32 = opt.f32;
    g.rows = rows;
    g.out = out;
    g.C = C;
    g.ldc = ldc;
    return g;
  }
  // The head on the listed rows of a block.  `pend`: the last residual sum and norm;
  // `row`: [width], `act`: [kLogitRows][ld_act], `out`: [kLogitRows][head.N].
  int logit_rows(NormRows pend, const Bf16Matrix &head, const int *rows, int n_rows, float *row,
                 void *act, float *out, float *dst) {
    int rc;
    BH_CHECK_HIP(hipMemcpyAsync(pf_pick, rows, sizeof(int) * n_rows, hipMemcpyHostToDevice, stream));
    if (n_rows == 1) {
      pend.rows = 1;
      pend.pick = pf_pick;
      pend.out_f32 = row;
      if ((rc = launch_norm_rows(pend, stream)))
        return rc;
      RowGemv g;
      g.W = head;
      g.src = row;
      g.out = logits;
      if ((rc = launch_row_gemv(g, stream)))
        return rc;
      if (dst != logits)
        BH_CHECK_HIP(hipMemcpyAsync(dst, logits, sizeof(float) * vocab, hipMemcpyDeviceToDevice, stream));
      return BUDDY_HIP_OK;
    }
    for (int r0 = 0; r0 < n_rows; r0 += kLogitRows) {
      const int m = std::min(kLogitRows, n_rows - r0);
      NormRows p = pend;
      p.rows = m;
      p.pick = pf_pick + r0;
      p.out_act = act;
      if ((rc = launch_norm_rows(p, stream)))
        return rc;
      if ((rc = launch_rows_gemm(gemm(head, act, p.ld_act, m, kOutF32, out, head.N), stream)))
        return rc;
      BH_CHECK_HIP(hipMemcpy2DAsync(dst + (size_t)r0 * vocab, sizeof(float) * vocab, out,
                                    sizeof(float) * head.N, sizeof(float) * vocab, m,
                                    hipMemcpyDeviceToDevice, stream));
    }
    return BUDDY_HIP_OK;
  }

  int prefill_rows(const int *tokens, int n, int start, const int *rows, int n_rows,
                   float *dst) override {
    int rc;
    if ((rc = seek(start)))
      return rc;
    if ((rc = ensure_block(std::min(n, opt.prefill_block))))
      return rc;
    next_pos = -1; // the device's position is the one of the last decode step
    int done_rows = 0;
    std::vector<int> local;
    for (int at = 0; at < n; at += opt.prefill_block) {
      const int m = std::min(opt.prefill_block, n - at);
      local.clear();
      while (done_rows + (int)local.size() < n_rows && rows[done_rows + local.size()] < at + m)
        local.push_back(rows[done_rows + local.size()] - at);
      BH_CHECK_HIP(hipMemcpyAsync(pf_tokens, tokens + at, sizeof(int) * m, hipMemcpyDefault, stream));
      if ((rc = run_block(m, start + at, local.data(), (int)local.size(),
                          dst ? dst + (size_t)done_rows * vocab : nullptr)))
        return rc;
      BH_CHECK_HIP(hipStreamSynchronize(stream)); // `local` is reused
      done_rows += (int)local.size();
      seq_len = start + at + m;
    }
    return BUDDY_HIP_OK;
  }
};

} // namespace bh
