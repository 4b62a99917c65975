// stack_model.hpp -- a decoder made of a list of layers, each a sequence mixer and an optional feed-forward, with norms ahead of
// and behind every sublayer.  The mechanisms are parameters (mixer kinds and their sizes, norm offset, layer scale, activations):
// a design fills a StackSpec and hands its tensors over (see lasapel.cpp), the stack owns the device layout, the caches and
// states of the live sequence, the launches of a step and of a prompt's portions.
//
//   x <- x + ls1 * norm1b(mixer(norm1(x)));  x <- x + ls2 * norm2b(ff(norm2(x)))
#pragma once

#include <memory>
#include <string>
#include <vector>

#include "sequence.hpp"

namespace bitnet_host {

struct RotarySpec {
    int dims = 0;
    double base = 10000.0;
    bool yarn = false;  // frequencies interpolated between f and f / factor, cos and sin scaled
    double factor = 1.0, original = 0.0, fast = 0.0, slow = 0.0;
    bool operator==(const RotarySpec &o) const {
        return dims == o.dims && base == o.base && yarn == o.yarn && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
};
// frequency of every pair and the factor on cos and sin
std::vector<double> rotary_frequencies(const RotarySpec &r, double *mult);

struct LatentSpec {  // attention over a shared latent (bitnet_hip_latent_*)
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;
    float scale = 1.f;
    RotarySpec rot;
    int kv_from = -1;  // the layer whose cache is read instead of one of its own
};
struct LinearSpec {  // linear attention with a constant decay per head (bitnet_hip_linear_*)
    int heads = 0, dim = 0, vdim = 0;
    std::vector<double> decay;
    int act_qkv = BITNET_HIP_ACT_SILU, act_gate = BITNET_HIP_ACT_SIGMOID;
};
struct LayerSpec {
    enum Mixer { Latent, Linear } mixer = Latent;
    LatentSpec latent;
    LinearSpec linear;
    int ff = 0;  // 0: no feed-forward
    int act_ff = BITNET_HIP_ACT_NONE;
};
struct StackSpec {
    int width = 0, vocab = 0;
    float eps = 1e-6f;
    float norm_offset = 0.f;  // block norms multiply by norm_offset + weight
    std::vector<LayerSpec> layers;
};

// One layer's tensors as the loader hands them over: bf16 matrices [out, in], f32 vectors.
struct StackLayerWeights {
    std::vector<float> norm1, norm1b, ls1, norm2, norm2b, ls2;  // empty ls: no layer scale
    const uint16_t *dq = nullptr, *uq = nullptr, *dkv = nullptr, *uk = nullptr, *uv = nullptr, *o = nullptr;
    std::vector<float> dq_norm, dkv_norm, sink;
    const uint16_t *q = nullptr, *k = nullptr, *v = nullptr, *g = nullptr;
    std::vector<float> out_norm;
    const uint16_t *up = nullptr, *down = nullptr;
    std::vector<float> up_b, down_b;
};

class StackModel : public Sequence {
  public:
    StackModel(const StackSpec &spec, bool f32, int max_pos);
    ~StackModel() override;

    int set_layer(int layer, const StackLayerWeights &w);
    int set_globals(const uint16_t *embed, const std::vector<float> &final_norm, const uint16_t *head);

    int prefill(int n, bool with_logits, int digits, float *elapsed_ms) override;
    int forward(const int32_t *tokens, int n, const int32_t *want, int n_want, float *logits) override;
    int last_hidden(float *out) override;
    size_t weight_bytes() const override { return weight_bytes_; }

  protected:
    bool ready() const override { return head_ != nullptr && layers_set_ == spec_.layers.size(); }
    int step(bool with_logits, int form) override;
    int clear_state() override;

  private:
    struct Matrix {
        uint16_t *w = nullptr;
        int rows = 0, cols = 0, ld = 0;  // cols: padded to a multiple of 8 for the matrix-vector product
    };
    struct Cache {  // one layer's latent cache
        void *c = nullptr, *r = nullptr;
    };
    struct Layer {
        float *norm1 = nullptr, *norm1b = nullptr, *ls1 = nullptr, *norm2 = nullptr, *norm2b = nullptr, *ls2 = nullptr;
        // latent
        int dimp = 0, rotp = 0, vdimp = 0, ldc = 0;
        Matrix down_q, uq, uk, uk_t, uv, o;  // down_q: dq, followed by dkv where the layer has one
        float *dq_norm = nullptr, *dkv_norm = nullptr, *sink = nullptr, *cos = nullptr, *sin = nullptr;
        Cache cache;
        // linear
        Matrix qkvg;
        float *out_norm = nullptr, *decay_pow = nullptr, *state = nullptr;
        // feed-forward
        Matrix up, down;
        float *up_b = nullptr, *down_b = nullptr;
        bool set = false;
    };
    struct Buffer {  // grown on demand, zero-filled: what a kernel reads past a matrix is finite
        void *p = nullptr;
        size_t bytes = 0;
    };
    // the sublayer whose output is still to be added to the residual stream
    struct Pending {
        const float *y = nullptr, *w = nullptr, *scale = nullptr;
    };

    int grow(Buffer &b, size_t bytes);
    template <class T>
    int upload(T **dst, const std::vector<T> &src);
    int upload_matrix(Matrix &m, const std::vector<uint16_t> &rows, int n_rows, int cols);
    int rope_tables(const RotarySpec &r, float **cos, float **sin);
    const Layer &kv_layer(size_t i) const { return layers_[spec_.layers[i].latent.kv_from >= 0 ? (size_t)spec_.layers[i].latent.kv_from : i]; }
    void attention_args(size_t i, bitnet_hip_latent_attention &a) const;
    void latent_args(size_t i, const float *z, size_t ldz, void *cq, size_t ldcq, bitnet_hip_latent_rows &r) const;
    // single token
    int gemv(const bitnet_hip_vector_input &in, const Matrix &m, const float *bias, int act0, int act1, size_t split, float *y,
             const bitnet_hip_latent_rows *latent = nullptr);
    bitnet_hip_vector_input block_input(const float *norm);
    int step_latent(size_t i);
    int step_linear(size_t i);
    // portion of n tokens
    int matmul(const void *a, size_t lda, bool a_f32, const Matrix &m, const float *bias, size_t n, int act0, int act1, size_t split, void *c, size_t ldc,
               bool c_f32);
    int portion(int n, int pos0);
    int portion_latent(size_t i, size_t n, size_t pos0);
    int portion_linear(size_t i, size_t n);
    int portion_buffers(size_t n);
    int set_position(int p);

    StackSpec spec_;
    bool f32_ = false;
    size_t cap_ = 0;  // positions the caches hold, a multiple of 64
    std::vector<Layer> layers_;
    size_t layers_set_ = 0;
    Matrix embed_, head_m_;
    const uint16_t *head_ = nullptr;
    float *final_norm_ = nullptr;
    size_t weight_bytes_ = 0;
    std::vector<void *> owned_;  // every fixed allocation
    struct RopeTable {
        RotarySpec spec;
        float *cos, *sin;
    };
    std::vector<RopeTable> ropes_;
    // single-token vectors (f32)
    float *x_[2] = {nullptr, nullptr}, *z_ = nullptr, *q_ = nullptr, *qabs_ = nullptr, *att_ = nullptr, *y_[2] = {nullptr, nullptr}, *act_ = nullptr,
          *lin_ = nullptr, *lino_ = nullptr, *scratch_ = nullptr;
    void *argmax_ = nullptr;
    int cur_ = 0;  // which x_ the step's residual stream is in
    Pending pending_;
    const float *hidden_ = nullptr;  // residual stream of the last position run
    // portion buffers; T = bf16, or f32 in 32-bit mode
    size_t rows_cap_ = 0;
    Buffer px_, ph_, pz_, pcq_, pq_, pqf_, pqabs_, patt_, py_, pact_, pk_, pvt_, plin_, plinf_, plino_, pgate_, pscratch_, plws_, pwant_, pxw_, phw_, plog_;
};

}  // namespace bitnet_host
