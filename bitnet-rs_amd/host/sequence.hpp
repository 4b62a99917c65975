// sequence.hpp -- what every model of this library shares above the C ABI: one live sequence (device token history, position,
// forced / sampled tokens), the step loop with its captured hipGraphs, and the interface a host drives
// (KVCache::clear, the greedy loop and the forced-token parity entry points of the reference: T:1251-1255,
// crates/bitnet-cli/src/main.rs:1282-1477, crates/bitnet-inference/src/parity.rs:30-111).
// A model supplies the launches of one step, and -- where it has one -- a many-token forward.
#pragma once

#include <cstddef>
#include <cstdint>
#include <string>

#include <hip/hip_runtime_api.h>

#include "bitnet_hip.h"

namespace bitnet_host {

struct Event {  // RAII: an error return between create and destroy must not leak the event
    hipEvent_t e = nullptr;
    ~Event() {
        if (e) hipEventDestroy(e);
    }
};

#define HCHK(expr)                                                                     \
    do {                                                                               \
        hipError_t _e = (expr);                                                        \
        if (_e != hipSuccess) {                                                        \
            char _b[256];                                                              \
            snprintf(_b, sizeof(_b), "HIP error %s at %s:%d (%s)", hipGetErrorName(_e), __FILE__, __LINE__, #expr); \
            err_ = _b;                                                                 \
            return BITNET_HIP_ERR_GPU;                                                 \
        }                                                                              \
    } while (0)
#define BCHK(expr)                       \
    do {                                 \
        int _rc = (expr);                \
        if (_rc != 0) return fail(#expr); \
    } while (0)

class Sequence {
  public:
    virtual ~Sequence();
    Sequence(const Sequence &) = delete;
    Sequence &operator=(const Sequence &) = delete;

    const std::string &error() const { return err_; }
    bool dead() const { return dead_; }  // construction failed: only error() and the destructor may be used
    void set_error(const std::string &e) { err_ = e; }
    int vocab() const { return vocab_; }
    int width() const { return width_; }
    int max_pos() const { return max_pos_; }

    // A new sequence: position 0, empty history, whatever the model carries from token to token cleared.
    int reset();
    // Put `n` forced tokens at the end of the history (the prompt).
    int feed(const int32_t *tokens, int n);
    // Run `n` single-token steps (T:1482-1504 body each).  with_logits=false skips the logits for positions nobody samples
    // from.  Uses the captured graph when use_graph, else eager launches.  Synchronises the stream before returning.
    virtual int run(int n, bool with_logits, bool use_graph, float *elapsed_ms);
    // The next n fed tokens as [n, *] matrices; with_logits samples the token after them exactly as run() does.
    // digits: fixed-point digits per activation, where the model's matmuls have such a choice.
    virtual int prefill(int n, bool with_logits, int digits, float *elapsed_ms) = 0;
    // The next n tokens of the sequence, forced; logits [n_want][vocab] (host) of the places `want` among them.
    virtual int forward(const int32_t *tokens, int n, const int32_t *want, int n_want, float *logits);
    // Captures and instantiates the step graph of every form a sequence can reach ahead of time, so that no run() pays for a
    // capture in the middle of a generation.  Nothing executes.
    int prepare_graphs(bool with_logits);
    int position();                    // tokens consumed so far
    int history(int32_t *out, int n);  // first n tokens of the sequence
    int last_logits(float *out);       // [vocab], of the last step run with logits
    virtual int last_hidden(float *out) = 0;  // residual stream after the last block (pre final norm)
    virtual size_t weight_bytes() const = 0;
    void *stream() const { return stream_; }

  protected:
    Sequence() = default;
    int init_sequence(int vocab, int width, int max_pos);  // stream, history, logits; sets err_ on failure
    int fail(const char *what);
    int fail_arg(const char *what);
    int check_run(int n, bool with_logits);
    int ensure_graph(bool with_logits, int form);
    void drop_graphs();

    virtual bool ready() const = 0;                            // weights are there
    virtual int step(bool with_logits, int form) = 0;          // the launches of one single-token step
    virtual int form_at(int) const { return 0; }               // which form of them a step at this position takes
    virtual int clear_state() { return 0; }

    bool dead_ = true;
    std::string err_;
    int vocab_ = 0, width_ = 0, max_pos_ = 0;
    void *stream_ = nullptr;
    float *logits_ = nullptr;
    int32_t *pos_ = nullptr, *n_forced_ = nullptr, *history_ = nullptr, *token_ = nullptr;
    int host_forced_ = 0;
    static constexpr int kForms = 3;
    void *graph_exec_[2 * kForms] = {};  // [2 * form + with_logits]
    void *graph_[2 * kForms] = {};
};

}  // namespace bitnet_host
