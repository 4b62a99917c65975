// stack_model.hpp -- a decoder made of a list of layers, each a sequence mixer and an optional feed-forward.  The mechanisms are
// parameters (mixer kinds and their sizes, kind and place of norms, layer scale, activations, experts, layers that run several times):
// a design fills a StackSpec and hands its tensors over (see lasapel.cpp, mimolix.cpp, lurepel.cpp, sipelorn.cpp), the stack owns the device layout, the caches and
// states of the live sequence, the launches of a step and of a prompt's portions.
//
//   one sublayer behind the other   x <- x + ls1 * norm1b(mixer(norm1(x)));  x <- x + ls2 * norm2b(ff(norm2(x)))
//   side by side                    x <- x + m * (mixer(norm1(x)) + ff(norm1(x)))
// (no norm behind a sublayer: m takes the place of ls * norm; no norm ahead of it: the sublayer reads x itself).  What a sublayer adds may be gated column by
// column from its input, and behind its sublayers a layer may add what the token itself brings along (a part of a table's row, weighed by x).  A loop runs a range of layers several times with the same weights, every
// pass with caches and states of its own and, ahead of its first layer, x <- W_in [x; embedding output].
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
    bool banded = false;  // f / factor for pairs of fewer than `slow` turns within the original length, f for more than `fast`, a line in between
    double factor = 1.0, original = 0.0, fast = 0.0, slow = 0.0;
    bool operator==(const RotarySpec &o) const {
        return dims == o.dims && base == o.base && yarn == o.yarn && banded == o.banded && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
};
// frequency of every pair and the factor on cos and sin
std::vector<double> rotary_frequencies(const RotarySpec &r, double *mult);

struct LatentSpec {  // attention over a shared latent (bitnet_hip_latent_*)
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;  // q_rank 0: queries straight from the layer's input
    bool neighbours = false;  // elements 2 i and 2 i + 1 turn together, not i and i + rot_dim / 2
    float scale = 1.f;
    RotarySpec rot;
    int kv_from = -1;  // the layer whose cache is read instead of one of its own
};
struct LinearSpec {  // linear attention with a constant decay per head (bitnet_hip_linear_*)
    int heads = 0, dim = 0, vdim = 0;
    std::vector<double> decay;
    int act_qkv = BITNET_HIP_ACT_SILU, act_gate = BITNET_HIP_ACT_SIGMOID;
};
struct AttentionSpec {  // keys and values of its own, shared by groups of query heads; one softmax map per head or two (bitnet_hip_gqa_*)
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, maps = 1;
    float scale = 1.f;
    double temp_coef = 0.0, temp_every = 1.0;  // a query at position p is multiplied by 1 + coef ln(floor((p + 1) / every) + 1)
    float diff = 0.f;                          // two maps: constant part of lambda, and 1 - diff scales the normed difference
    RotarySpec rot;                            // dims 0: none; neighbouring elements turn together
    int chunk = 0;                             // positions see their own chunk only; 0: everything ahead of them
    bool unit_norm = false;                    // queries and keys divided by their root mean square
    bool values_are_keys = false;              // no values of their own
    bool head_gate = false;                    // a factor per head from the layer's input
    bool column_gate = false;                  // a factor per column of the heads' outputs
    int window = 0;                            // a position sees itself and the window - 1 positions ahead of it; 0: no window
    bool far_penalty = false;                  // weight ln(1 + rate * distance) taken off a score, two numbers per head
    int taps = 0;                              // queries, keys and values pass a causal convolution over that many positions; 0: none
    int kv_from = -1;                          // the layer whose keys and values are read instead of ones of its own
};
struct DeltaSpec {  // gated delta rule (bitnet_hip_delta_*)
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 1;
    float unit_eps = 1e-6f;
};
struct ExpertsSpec {  // routed experts (bitnet_hip_experts_*); count 0: none
    int count = 0, top = 0, ff = 0, act = BITNET_HIP_ACT_NONE;
    float scale = 1.f;
    bool raw = false;    // weights as the scores are, not divided by the chosen ones' sum
    bool gated = false;  // act(gate) * up
    int identity = 0;    // experts behind these whose output is their input
    bool sigmoid = false;        // scores: every logit by itself, not a softmax
    int groups = 0, keep = 0;    // choice among the experts of the best `keep` of `groups` groups of neighbours; 0: among all
};
struct LayerSpec {
    enum Mixer { Latent, Linear, Attention, Delta } mixer = Latent;
    LatentSpec latent;
    LinearSpec linear;
    AttentionSpec attention;
    DeltaSpec delta;
    bool parallel = false;  // mixer and feed-forward side by side behind one norm (attention and delta mixers)
    int ff = 0;             // every token's feed-forward: dense, or the expert shared by all; 0: none
    int act_ff = BITNET_HIP_ACT_NONE;
    bool gated = false;     // act_ff(gate) * up
    bool shared_gate = false;  // the expert shared by all is multiplied by a number per token (not side by side with a mixer)
    ExpertsSpec experts;
};
struct LoopSpec {  // layers start .. stop - 1 run `times` times in a row
    int start = 0, stop = 0, times = 0;  // times 0: no loop
};
struct PairsSpec {  // a second embedding, of the previous and the current token: row (prev * mul_prev + cur * mul_cur) mod buckets; the first token: row `buckets`
    uint64_t buckets = 0, mul_prev = 0, mul_cur = 0;  // buckets 0: none
};
struct StackSpec {
    int width = 0, vocab = 0;
    float eps = 1e-6f;
    float norm_offset = 0.f;     // block norms multiply by norm_offset + weight
    bool center = false;         // block norms are layer norms, with a bias
    float embed_scale = 1.f;
    float residual_mult = 1.f;   // on a sublayer without a norm behind it
    bool residual_gate = false;  // what a sublayer adds is multiplied by sigmoid(W h + b), h being its input
    PairsSpec pairs;
    int side_dim = 0;            // columns of the table of token inputs per layer; 0: no such inputs
    LoopSpec loop;
    std::vector<LayerSpec> layers;
};

// One layer's tensors as the loader hands them over: bf16 matrices [out, in], f32 vectors.
struct StackLayerWeights {
    std::vector<float> norm1, norm1b, ls1, norm2, norm2b, ls2;  // empty ls: no layer scale; other empty ones: no norm ahead of, behind the sublayer
    std::vector<float> norm1_bias, norm2_bias;
    const uint16_t *dq = nullptr, *uq = nullptr, *dkv = nullptr, *uk = nullptr, *uv = nullptr, *o = nullptr;
    std::vector<float> dq_norm, dkv_norm, sink;
    const uint16_t *q = nullptr, *k = nullptr, *v = nullptr, *g = nullptr;
    std::vector<float> out_norm;
    std::vector<float> q_norm, k_norm, lq1, lk1, lq2, lk2;              // attention; empty q_norm, k_norm: no norm
    const uint16_t *b = nullptr, *a = nullptr;                          // delta: step size and decay, one row per head
    std::vector<float> q_conv, k_conv, v_conv, a_log, dt_bias;          // [channels][taps]
    const uint16_t *gate = nullptr, *up = nullptr, *down = nullptr, *router = nullptr;
    std::vector<float> up_b, down_b, router_correction;                  // empty correction: none
    std::vector<const uint16_t *> expert_gate, expert_up, expert_down;
    std::vector<float> q_b, k_b, v_b, far_weight, far_rate;              // attention; empty biases: none
    const uint16_t *rg1 = nullptr, *rg2 = nullptr;                       // residual gates [width, width]
    std::vector<float> rg1_b, rg2_b;
    float act_a = 0.f, act_b = 0.f;                                      // constants of act_ff
    const uint16_t *shared_gate = nullptr;                               // [1, width]
    const uint16_t *side_gate = nullptr, *side_proj = nullptr;           // [side_dim, width], [width, side_dim]
    std::vector<float> side_norm;
};
struct StackGlobalWeights {
    const uint16_t *embed = nullptr, *head = nullptr, *loop_in = nullptr;
    const uint16_t *pairs = nullptr;  // [buckets + 1, width]
    const uint16_t *side = nullptr;   // [vocab, layers * side_dim]
    std::vector<float> final_norm, final_bias, embed_norm;  // empty bias, norm behind the embedding: none
};

class StackModel : public Sequence {
  public:
    StackModel(const StackSpec &spec, bool f32, int max_pos);
    ~StackModel() override;

    int set_layer(int layer, const StackLayerWeights &w);
    int set_globals(const StackGlobalWeights &w);

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
    struct Slot {  // what one pass of a layer carries from token to token
        void *c = nullptr, *r = nullptr;       // latent: rows, rotated parts
        void *k = nullptr, *v = nullptr;       // attention: keys, transposed values
        float *state = nullptr, *ring = nullptr;  // linear, delta: state; delta, attention: the last inputs of the convolution
        size_t state_bytes = 0;
    };
    struct Norm {
        float *w = nullptr, *bias = nullptr;
    };
    // Sublayers that read one norm and whose outputs add up, as two products and what lies between them.  A row of activations is
    // [mixer output, ko | feed-forward, fs | residual gate, rg | the mixer's projections, main]; `in` makes everything behind the mixer's output from the
    // normed row (and the tail: rows whose results stay f32 in a prompt -- the shared expert's number, the mixer's, the router's), `out` takes the first
    // ko + fs columns back to the residual stream.
    struct Block {
        bool used = false, mixer = false;
        bool gated = false;  // the feed-forward's rows of `in` come in pairs
        Norm norm;
        Matrix in, out, expert_up, expert_down;
        int ko = 0, fs = 0, rg = 0, main = 0, tail = 0, gates = 0;  // gates: rows of the tail ahead of the router
        int shared = 0;                                             // 1: the tail's first row is the shared expert's number
        int ff_rows() const { return gated ? 2 * fs : fs; }
        float *in_bias = nullptr, *out_bias = nullptr;
    };
    struct Layer {
        Norm norm1, norm2;
        float *norm1b = nullptr, *ls1 = nullptr, *norm2b = nullptr, *ls2 = nullptr;
        std::vector<Slot> slots;  // one per pass
        Block block[2];
        // attention
        float *q_norm = nullptr, *k_norm = nullptr, *q_factor = nullptr;
        float lambda = 0.f;
        int gate_at = 0;  // where a row of projections holds the heads' gates
        int channels = 0;  // columns of it that a convolution covers
        float *far_weight = nullptr, *far_rate = nullptr;
        // experts
        float *correction = nullptr;
        // delta
        float *conv = nullptr /* attention too */, *decay_rate = nullptr, *dt_bias = nullptr;
        // latent
        int dimp = 0, rotp = 0, vdimp = 0, ldc = 0;
        Matrix down_q, uq, uk, uk_t, uv, o;  // down_q: dq, followed by dkv where the layer has one
        float *dq_norm = nullptr, *dkv_norm = nullptr, *sink = nullptr, *cos = nullptr, *sin = nullptr;
        // linear (out_norm: delta too)
        Matrix qkvg;
        float *out_norm = nullptr, *decay_pow = nullptr;
        // feed-forward
        Matrix up, down;
        float *up_b = nullptr, *down_b = nullptr;
        float act_a = 0.f, act_b = 0.f;
        // token input
        Matrix side_gate, side_proj;
        float *side_norm = nullptr;
        bool set = false;
    };
    struct Buffer {  // grown on demand, zero-filled: what a kernel reads past a matrix is finite
        void *p = nullptr;
        size_t bytes = 0;
    };
    // the sublayer whose output is still to be added to the residual stream
    struct Pending {
        const float *y = nullptr, *w = nullptr, *scale = nullptr;
        const void *gate = nullptr;   // one token: f32; a portion: rows of ld_gate, of the activations' type
        size_t ld_gate = 0;
        const float *y_scale = nullptr;  // a portion: a number per row on y, ld_y_scale apart
        size_t ld_y_scale = 0;
        bool experts = false;         // a portion's routed rows join in (y may be missing)
        const void *input = nullptr;  // what those experts read, if not the residual stream
        bool identity = false;        // some of them hand it through
    };
    struct Run {
        size_t layer;
        int pass;
        bool enters;  // the first layer of a pass of the loop
    };

    int grow(Buffer &b, size_t bytes);
    template <class T>
    int upload(T **dst, const std::vector<T> &src);
    int upload_matrix(Matrix &m, const std::vector<uint16_t> &rows, int n_rows, int cols);
    int rope_tables(const RotarySpec &r, float **cos, float **sin);
    int query_factors(const AttentionSpec &a, float **out);
    int embed_rows(size_t n, float *out);
    bitnet_hip_router router_args(size_t i) const;
    int plan_runs();
    int plan_block(size_t i, int which, bool mixer, bool ff);
    bool alloc(void **p, size_t bytes);
    int set_block(size_t i, int which, const StackLayerWeights &w);
    const Slot &kv_slot(size_t i, int pass) const {
        const LayerSpec &S = spec_.layers[i];
        const int from = S.mixer == LayerSpec::Latent ? S.latent.kv_from : S.mixer == LayerSpec::Attention ? S.attention.kv_from : -1;
        return layers_[from >= 0 ? (size_t)from : i].slots[(size_t)pass];
    }
    bool fits_source(size_t i) const;
    int set_latent(Layer &L, const LatentSpec &m, const StackLayerWeights &w);
    void attention_args(size_t i, int pass, bitnet_hip_latent_attention &a) const;
    void latent_args(size_t i, int pass, const float *z, size_t ldz, void *cq, size_t ldcq, bitnet_hip_latent_rows &r) const;
    bitnet_hip_gqa gqa_args(size_t i, int pass, const void *proj, size_t ld, bool f32) const;
    bitnet_hip_delta delta_args(size_t i, int pass) const;
    // single token
    int gemv(const bitnet_hip_vector_input &in, const Matrix &m, const float *bias, int act0, int act1, size_t split, float *y,
             const bitnet_hip_latent_rows *latent = nullptr, const bitnet_hip_epilogue *more = nullptr);
    bitnet_hip_vector_input block_input(const Norm &norm);
    void add_pending(bitnet_hip_vector_input &in);
    int step_latent(size_t i, int pass);
    int step_attend_latent(size_t i, int pass, const float *q, const bitnet_hip_latent_rows *rows, float *out, size_t ldo);
    int step_side(size_t i);
    int step_linear(size_t i, int pass);
    int step_block(size_t i, int pass, int which);
    int step_loop_in();
    // portion of n tokens
    int matmul(const void *a, size_t lda, bool a_f32, const Matrix &m, const float *bias, size_t n, int act0, int act1, size_t split, void *c, size_t ldc,
               bool c_f32, const bitnet_hip_epilogue *more = nullptr);
    int block_matmul(const Layer &L, const Block &B, int first, int rows, size_t n, int act0, int act1, int split, void *c, size_t ldc, bool c_f32);
    int portion(int n, int pos0);
    int portion_norm(size_t n, const Norm *norm, const float *x2, void *h, size_t ldh);
    int portion_latent(size_t i, int pass, size_t n, size_t pos0);
    int portion_attend_latent(size_t i, int pass, size_t n, size_t pos0, const uint16_t *q, const float *qf, size_t ldq, void *out, size_t ldo);
    int portion_side(size_t i, size_t n);
    int portion_linear(size_t i, int pass, size_t n);
    int portion_block(size_t i, int pass, int which, size_t n, size_t pos0);
    int portion_loop_in(size_t n);
    int portion_buffers(size_t n);
    int set_position(int p);

    StackSpec spec_;
    bool f32_ = false;
    size_t cap_ = 0;  // positions the caches hold, a multiple of 128
    std::vector<Layer> layers_;
    std::vector<Run> runs_;
    size_t layers_set_ = 0;
    Matrix embed_, head_m_, loop_in_, pairs_, side_;
    const uint16_t *head_ = nullptr;
    Norm final_norm_;
    float *embed_norm_ = nullptr;
    size_t weight_bytes_ = 0;
    std::vector<void *> owned_;  // every fixed allocation
    struct RopeTable {
        RotarySpec spec;
        float *cos, *sin;
    };
    std::vector<RopeTable> ropes_;
    // single-token vectors (f32); x0_: the embedding output
    float *x0_ = nullptr, *row_[2] = {nullptr, nullptr}, *h_ = nullptr, *eact_ = nullptr;
    int32_t *eids_ = nullptr;
    float *x_[2] = {nullptr, nullptr}, *z_ = nullptr, *q_ = nullptr, *qabs_ = nullptr, *att_ = nullptr, *y_[2] = {nullptr, nullptr}, *act_ = nullptr,
          *lin_ = nullptr, *lino_ = nullptr, *scratch_ = nullptr;
    void *argmax_ = nullptr;
    int row_at_ = 0;  // the row the last block used: its residual gate is read while the next block's is written
    const float *cur_ = nullptr;  // where the step's residual stream is
    float *next_x() const { return cur_ == x_[0] ? x_[1] : x_[0]; }
    Pending pending_;
    const float *hidden_ = nullptr;  // residual stream of the last position run
    // portion buffers; T = bf16, or f32 in 32-bit mode
    size_t rows_cap_ = 0;
    Buffer px_, ph_, pz_, pcq_, pq_, pqf_, pqabs_, patt_, py_, pact_, pk_, pvt_, plin_, plinf_, plino_, pgate_, pscratch_, plws_, pwant_, pxw_, phw_, plog_;
    Buffer px0_, pcat_, prow_, ptail_, pqk_, pv_, pgates_, pplan_, peact_, peout_, pqc_;
    bitnet_hip_experts_plan plan_;
};

}  // namespace bitnet_host
