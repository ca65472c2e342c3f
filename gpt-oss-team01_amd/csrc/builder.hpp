// Loading weights: host payloads through pinned double-buffered staging (or on-device random
// weights) into the kernels' device layouts.
#pragma once
#include <string.h>

#include <system_error>
#include <thread>

#include "engine.hpp"

namespace gptoss {

// Host -> device staging of the fp32 payload: two pinned host buffers and two device buffers.
// Chunk i is copied by the host into pinned[i % 2] (several threads), sent with an asynchronous
// copy on its own stream, and converted/packed by a kernel on the engine's stream; the copy of chunk
// i+1 and the host's work on chunk i+2 overlap that kernel.  Events order the reuse of either
// buffer; the host only ever waits for the copy issued two chunks earlier.  Replaces the host-side
// transposes and synchronous uploads of getp-csrc/src/alloc.cpp:27-35,112-127.
struct Stager {
  hipStream_t copy = nullptr;
  float *pinned[2] = {nullptr, nullptr}, *dev[2] = {nullptr, nullptr};
  hipEvent_t h2d_done[2] = {nullptr, nullptr}, consumed[2] = {nullptr, nullptr};
  size_t elems = 0;   // floats per buffer
  unsigned next = 0;
};

// plain copy by a few threads: one thread reaches a fraction of what the host memory can deliver
inline void host_copy(float *dst, const float *src, size_t n) {
  constexpr int T = 6;
  if (n < ((size_t)1 << 20)) {
    memcpy(dst, src, n * sizeof(float));
    return;
  }
  std::thread th[T - 1];
  const size_t per = (n + T - 1) / T;
  int started = 0;
  for (int i = 1; i < T; i++) {
    const size_t lo = std::min(n, per * i), hi = std::min(n, per * (i + 1));
    try {
      th[i - 1] = std::thread([=] { memcpy(dst + lo, src + lo, (hi - lo) * sizeof(float)); });
      started = i;
    } catch (const std::system_error &) {
      break;  // no more threads to be had (a thread or pid limit): this thread copies the rest
    }
  }
  memcpy(dst, src, std::min(n, per) * sizeof(float));
  const size_t rest = std::min(n, per * (size_t)(started + 1));
  if (rest < n) memcpy(dst + rest, src + rest, (n - rest) * sizeof(float));
  for (int i = 1; i <= started; i++) th[i - 1].join();
}

struct Builder {
  gptoss_engine *e;
  int rc = GPTOSS_OK;
  Stager st;                      // fp32 payload on its way to the device (host weights only)
  bf16_t *stage_bf16 = nullptr;   // synthetic weights before packing
  size_t stage_elems = 0;
  // MXFP4 expert storage: unpacked codes and scales of one staging chunk, and the flag the
  // requantisation kernel raises when a value has no exact MXFP4 representation
  unsigned char *q_blocks = nullptr, *q_scales = nullptr;
  int *q_not_exact = nullptr;

  template <typename T>
  T *alloc(size_t n) {
    if (rc != GPTOSS_OK) return nullptr;
    void *p = nullptr;
    size_t bytes = align_up(std::max<size_t>(n, 1) * sizeof(T), 256);
    hipError_t err = hipMalloc(&p, bytes);
    if (err != hipSuccess) {
      rc = fail(GPTOSS_ERR_HIP, "engine: hipMalloc of %zu bytes failed: %s", bytes, hipGetErrorString(err));
      return nullptr;
    }
    e->allocs.push_back(p);
    e->device_bytes += bytes;
    return (T *)p;
  }

  bool ok() const { return rc == GPTOSS_OK; }
  void check(int r) { if (rc == GPTOSS_OK && r != GPTOSS_OK) rc = r; }
  void hip(hipError_t err, const char *what) {
    if (rc == GPTOSS_OK && err != hipSuccess) rc = fail(GPTOSS_ERR_HIP, "engine: %s: %s", what, hipGetErrorString(err));
  }

  void stager_create(size_t elems) {
    st.elems = elems;
    hip(hipStreamCreate(&st.copy), "hipStreamCreate");
    for (int i = 0; i < 2 && ok(); i++) {
      hip(hipHostMalloc((void **)&st.pinned[i], elems * sizeof(float), hipHostMallocDefault), "staging hipHostMalloc");
      hip(hipMalloc((void **)&st.dev[i], elems * sizeof(float)), "staging hipMalloc");
      hip(hipEventCreateWithFlags(&st.h2d_done[i], hipEventDisableTiming), "hipEventCreate");
      hip(hipEventCreateWithFlags(&st.consumed[i], hipEventDisableTiming), "hipEventCreate");
    }
  }
  void stager_destroy() {
    if (st.copy) (void)hipStreamSynchronize(st.copy);
    for (int i = 0; i < 2; i++) {
      if (st.pinned[i]) (void)hipHostFree(st.pinned[i]);
      if (st.dev[i]) (void)hipFree(st.dev[i]);
      if (st.h2d_done[i]) (void)hipEventDestroy(st.h2d_done[i]);
      if (st.consumed[i]) (void)hipEventDestroy(st.consumed[i]);
    }
    if (st.copy) (void)hipStreamDestroy(st.copy);
    st = Stager();
  }
  // n floats of the payload -> a device buffer the engine's stream may read once this returns (the
  // wait is enqueued, not performed); release(slot) after the kernels that read it are enqueued
  const float *stage_in(const float *host, size_t n, int *slot) {
    const int sl = (int)(st.next++ & 1);
    *slot = sl;
    if (!ok()) return nullptr;
    // pinned[sl] is free once the copy that last read it has finished (an event never recorded is complete)
    hip(hipEventSynchronize(st.h2d_done[sl]), "hipEventSynchronize");
    if (!ok()) return nullptr;
    host_copy(st.pinned[sl], host, n);
    // dev[sl] is free once the kernels that last read it have finished
    hip(hipStreamWaitEvent(st.copy, st.consumed[sl], 0), "hipStreamWaitEvent");
    hip(hipMemcpyAsync(st.dev[sl], st.pinned[sl], n * sizeof(float), hipMemcpyHostToDevice, st.copy), "H2D");
    hip(hipEventRecord(st.h2d_done[sl], st.copy), "hipEventRecord");
    hip(hipStreamWaitEvent(e->stream, st.h2d_done[sl], 0), "hipStreamWaitEvent");
    return st.dev[sl];
  }
  void release(int slot) { hip(hipEventRecord(st.consumed[slot], e->stream), "hipEventRecord"); }

  // fp32 host tensor -> fp32 device tensor
  float *upload_f32(const float *host, size_t n, uint64_t seed, float mean, float std) {
    float *d = alloc<float>(n);
    if (!ok()) return nullptr;
    if (!host) {
      check(run_synth_f32(d, n, seed, mean, std, e->stream));
      return d;
    }
    for (size_t o = 0; o < n && ok(); o += st.elems) {
      const size_t c = std::min(st.elems, n - o);
      int slot;
      const float *src = stage_in(host + o, c, &slot);
      if (!ok()) break;
      hip(hipMemcpyAsync(d + o, src, c * sizeof(float), hipMemcpyDeviceToDevice, e->stream), "D2D");
      release(slot);
    }
    return d;
  }

  // fp32 host matrices -> bf16 device matrices, row-major (pack == false) or fragment order
  bf16_t *upload_matrices(const float *host, int n_mat, int n_out, int n_in, bool pack, int pack_flags,
                          uint64_t seed, float std) {
    size_t per = (size_t)n_out * n_in;
    bf16_t *dst = alloc<bf16_t>(per * n_mat);
    if (!ok()) return nullptr;
    if (per > stage_elems) {
      rc = fail(GPTOSS_ERR_DIM, "engine: a %d x %d matrix exceeds the staging buffer", n_out, n_in);
      return nullptr;
    }
    int group = (int)std::max<size_t>(1, stage_elems / per);
    for (int m0 = 0; m0 < n_mat && ok(); m0 += group) {
      int nm = std::min(group, n_mat - m0);
      size_t n = per * nm;
      if (host) {
        int slot;
        const float *src = stage_in(host + per * m0, n, &slot);
        if (!ok()) break;
        if (pack) check(gptoss_pack_weight(src, dst + per * m0, nm, n_out, n_in, pack_flags | GPTOSS_PACK_SRC_FP32, e->stream));
        else check(run_f32_to_bf16(src, dst + per * m0, n, e->stream));
        release(slot);
      } else {
        // one stream, in order: the staging buffer is rewritten only after the kernel that read it
        check(run_synth_bf16(stage_bf16, n, seed + 7919ull * (uint64_t)m0, 0.f, std, e->stream));
        if (!ok()) break;
        if (pack) check(gptoss_pack_weight(stage_bf16, dst + per * m0, nm, n_out, n_in, pack_flags, e->stream));
        else hip(hipMemcpyAsync(dst + per * m0, stage_bf16, n * sizeof(bf16_t), hipMemcpyDeviceToDevice, e->stream), "D2D");
      }
    }
    return dst;
  }

  // fp32 host matrices (exactly MXFP4-representable) or random MXFP4 weights -> packed MXFP4
  bf16_t *upload_matrices_mxfp4(const float *host, int n_mat, int n_out, int n_in, int pack_flags,
                                uint64_t seed) {
    const size_t per = (size_t)n_out * n_in;
    const size_t mat_bytes = per / 2 + per / 32;
    unsigned char *dst = alloc<unsigned char>(mat_bytes * n_mat);
    if (!ok()) return nullptr;
    if (per > stage_elems) {
      rc = fail(GPTOSS_ERR_DIM, "engine: a %d x %d matrix exceeds the staging buffer", n_out, n_in);
      return nullptr;
    }
    const int group = (int)std::max<size_t>(1, stage_elems / per);
    for (int m0 = 0; m0 < n_mat && ok(); m0 += group) {
      const int nm = std::min(group, n_mat - m0);
      const size_t n_blocks = per * nm / 32;
      if (host) {
        int slot;
        const float *src = stage_in(host + per * m0, per * nm, &slot);
        if (!ok()) break;
        check(run_requant_mxfp4(src, n_blocks, q_blocks, q_scales, q_not_exact, e->stream));
        release(slot);
      } else {
        // scale exponents -13..-5: weights of the order of 0.02, as the bf16 synthetic weights
        check(run_synth_mxfp4(q_blocks, q_scales, n_blocks, seed + 7919ull * (uint64_t)m0, -5, e->stream));
      }
      if (!ok()) break;
      check(gptoss_pack_mxfp4(q_blocks, q_scales, dst + mat_bytes * m0, nm, n_out, n_in, pack_flags, e->stream));
    }
    return reinterpret_cast<bf16_t *>(dst);
  }
};

}  // namespace gptoss
