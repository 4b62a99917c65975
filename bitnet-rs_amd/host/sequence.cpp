// sequence.cpp -- see sequence.hpp.
#include "sequence.hpp"

#include <cstdio>
#include <vector>

namespace bitnet_host {

int Sequence::fail_arg(const char *what) {
    err_ = what;
    return BITNET_HIP_ERR_INVALID_ARGUMENT;
}

int Sequence::fail(const char *what) {
    const char *e = bitnet_hip_get_last_error();
    err_ = std::string(what) + ": " + (e ? e : "error");
    return BITNET_HIP_ERR_EXECUTION;
}

int Sequence::init_sequence(int vocab, int width, int max_pos) {
    vocab_ = vocab, width_ = width, max_pos_ = max_pos;
    BCHK(bitnet_hip_init(-1));
    hipStream_t s;
    HCHK(hipStreamCreateWithFlags(&s, hipStreamNonBlocking));
    stream_ = s;
    HCHK(hipMalloc((void **)&logits_, (size_t)vocab * 4));
    HCHK(hipMalloc((void **)&pos_, 4));
    HCHK(hipMalloc((void **)&n_forced_, 4));
    HCHK(hipMalloc((void **)&token_, 4));
    HCHK(hipMalloc((void **)&history_, ((size_t)max_pos + 2) * 4));
    return 0;
}

Sequence::~Sequence() {
    drop_graphs();
    for (void *p : {(void *)logits_, (void *)pos_, (void *)n_forced_, (void *)history_, (void *)token_})
        if (p) hipFree(p);
    if (stream_) hipStreamDestroy((hipStream_t)stream_);
}

void Sequence::drop_graphs() {
    for (int i = 0; i < 2 * kForms; ++i) {
        if (graph_exec_[i]) hipGraphExecDestroy((hipGraphExec_t)graph_exec_[i]);
        if (graph_[i]) hipGraphDestroy((hipGraph_t)graph_[i]);
        graph_exec_[i] = graph_[i] = nullptr;
    }
}

int Sequence::reset() {
    host_forced_ = 0;
    HCHK(hipMemset(pos_, 0, 4));
    HCHK(hipMemset(n_forced_, 0, 4));
    HCHK(hipMemset(history_, 0, ((size_t)max_pos_ + 2) * 4));
    return clear_state();
}

int Sequence::feed(const int32_t *tokens, int n) {
    const int p = position();
    if (p < 0) return BITNET_HIP_ERR_GPU;
    const int base = p > host_forced_ ? p : host_forced_;
    if (n < 0 || (n > 0 && !tokens)) return fail_arg("feed: null tokens");
    for (int i = 0; i < n; ++i)
        if (tokens[i] < 0 || tokens[i] >= vocab_) {  // TransformerModel::embed's index_select fails on it (T:1390-1426)
            char b[96];
            snprintf(b, sizeof(b), "token id %d out of range [0, %d)", tokens[i], vocab_);
            return fail_arg(b);
        }
    if (base + n > max_pos_) return fail_arg("KV cache overflow");  // T:1190-1194
    HCHK(hipMemcpy(history_ + base, tokens, (size_t)n * 4, hipMemcpyHostToDevice));
    host_forced_ = base + n;
    HCHK(hipMemcpy(n_forced_, &host_forced_, 4, hipMemcpyHostToDevice));
    return 0;
}

int Sequence::position() {
    int p = -1;
    if (hipMemcpy(&p, pos_, 4, hipMemcpyDeviceToHost) != hipSuccess) {
        err_ = "position readback failed";
        return -1;
    }
    return p;
}

int Sequence::history(int32_t *out, int n) {
    if (!out || n < 0 || n > max_pos_ + 2) return fail_arg("history: n out of range");
    HCHK(hipMemcpy(out, history_, (size_t)n * 4, hipMemcpyDeviceToHost));
    return 0;
}

int Sequence::last_logits(float *out) {
    HCHK(hipMemcpy(out, logits_, (size_t)vocab_ * 4, hipMemcpyDeviceToHost));
    return 0;
}

int Sequence::prepare_graphs(bool with_logits) {
    if (!ready()) return fail_arg("model globals not set");
    unsigned forms = 0;
    for (int pos = 0; pos + 1 < max_pos_; ++pos) forms |= 1u << form_at(pos);
    for (int f = 0; f < kForms; ++f)
        if (forms & (1u << f))
            if (int rc = ensure_graph(with_logits, f)) return rc;
    return 0;
}

int Sequence::ensure_graph(bool with_logits, int form) {
    const int gi = 2 * form + (with_logits ? 1 : 0);
    if (graph_exec_[gi]) return 0;
    hipStream_t s = (hipStream_t)stream_;
    hipGraph_t g = nullptr;
    HCHK(hipStreamBeginCapture(s, hipStreamCaptureModeGlobal));
    const int rc = step(with_logits, form);
    const hipError_t e = hipStreamEndCapture(s, &g);
    if (rc != 0) {
        if (g) hipGraphDestroy(g);
        return rc;
    }
    HCHK(e);
    hipGraphExec_t ex = nullptr;
    HCHK(hipGraphInstantiate(&ex, g, nullptr, nullptr, 0));
    graph_[gi] = g;
    graph_exec_[gi] = ex;
    return 0;
}

int Sequence::check_run(int n, bool with_logits) {
    if (!ready()) return fail_arg("model globals not set");
    const int p = position();
    if (p < 0) return BITNET_HIP_ERR_GPU;
    if (n < 0 || p + n > max_pos_ - 1) return fail_arg("KV cache overflow");  // T:1190-1194
    // a step without logits samples nothing: the NEXT position's token must already be in the history
    if (!with_logits && p + n > host_forced_) return fail_arg("run(with_logits = false) past the fed tokens: nothing would choose the next token");
    return 0;
}

int Sequence::run(int n, bool with_logits, bool use_graph, float *elapsed_ms) {
    if (int rc = check_run(n, with_logits)) return rc;
    const int p = position();
    hipStream_t s = (hipStream_t)stream_;
    if (use_graph) {
        for (int i = 0; i < n; ++i) {  // every form this run needs (at most three captures)
            int rc = ensure_graph(with_logits, form_at(p + i));
            if (rc) return rc;
        }
    }
    Event ev0, ev1;
    HCHK(hipEventCreate(&ev0.e));
    HCHK(hipEventCreate(&ev1.e));
    HCHK(hipEventRecord(ev0.e, s));
    for (int i = 0; i < n; ++i) {
        if (use_graph) {
            HCHK(hipGraphLaunch((hipGraphExec_t)graph_exec_[2 * form_at(p + i) + (with_logits ? 1 : 0)], s));
        } else {
            int rc = step(with_logits, form_at(p + i));
            if (rc) return rc;
        }
    }
    HCHK(hipEventRecord(ev1.e, s));
    HCHK(hipStreamSynchronize(s));
    float ms = 0.f;
    HCHK(hipEventElapsedTime(&ms, ev0.e, ev1.e));
    if (elapsed_ms) *elapsed_ms = ms;
    return 0;
}

int Sequence::forward(const int32_t *tokens, int n, const int32_t *want, int n_want, float *logits) {
    if (n_want < 0 || (n_want > 0 && (!want || !logits))) return fail_arg("forward: null pointer");
    for (int w = 0; w < n_want; ++w)
        if (want[w] < 0 || want[w] >= n) return fail_arg("forward: a wanted place is not among the tokens");
    if (int rc = feed(tokens, n)) return rc;
    for (int i = 0; i < n; ++i) {
        bool wanted = false;
        for (int w = 0; w < n_want; ++w) wanted = wanted || want[w] == i;
        if (int rc = run(1, wanted, true, nullptr)) return rc;
        for (int w = 0; w < n_want; ++w)
            if (want[w] == i)
                if (int rc = last_logits(logits + (size_t)w * vocab_)) return rc;
    }
    return 0;
}

}  // namespace bitnet_host
