// A mixer with a matrix memory instead of keys and values.
//
//   mlstm   per head q = q_scale W_q x and k = W_k x of head_dim elements, v = W_v x of value_dim; an input gate and a forget gate per
//           head and token, kept as logarithms: a = c tanh((w_i x + b_i) / c), f = log sigmoid(c tanh((w_f x + b_f) / c)), c the cap.
//           With a running maximum m_t = max(f_t + m_(t-1), a_t) from zero:
//             S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(a - m_t) k_t v_t^T,   n_t the same with k_t alone,
//             o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6).
//           Each head's o is divided by its root mean square, the heads side by side are multiplied by a weight over all their elements
//           and by sigmoid(W_g x), and W_o projects back.
//
// The state of a sequence is one float32 row of the cache's state groups (zero when a slot is taken): per head S and n one behind the
// other, then the heads' m.  Gates, maxima, n, S and the heads' norm are float32 whatever the activation type, and so are the gates'
// products' results; q, k, v, the output gate and the gates come from one product with the weights stacked.  Steps that bring many tokens of a
// sequence in bfloat16 run in chunks on the matrix cores (mlstm.hip), with the heads' norm and the gate in the last of their kernels.
//
// params: hidden, heads, head_dim, value_dim, gate_cap, eps; optional q_scale (head_dim^(-1/2) unless given), names {q, k, v, g, o, norm, i,
// i_bias, f, f_bias}.
#include <math.h>

#include "kernels.h"
#include "linear.h"
#include "parts.h"
#include "step.h"

namespace tq {
namespace {

OwnedPtr take(Loaded& tensors, const std::string& name) {
    auto it = tensors.find(name);
    if (it == tensors.end() || !it->second) raise(TQE_ERR_WEIGHTS, "a part was not given its tensor '%s'", name.c_str());
    return it->second;
}

OwnedPtr as_floats(const OwnedPtr& p, hipStream_t stream) {
    if (p->t.dtype == F32) return p;
    std::vector<int64_t> dims(p->t.shape, p->t.shape + p->t.ndim);
    OwnedPtr out = make_owned(F32, dims);
    if (!null_device()) K::convert(p->t.data, p->t.dtype, out->t.data, F32, (long long)p->t.numel(), stream);
    stream_synchronize(stream);
    return out;
}

const void* at(const Tensor& t, int64_t column) { return (const char*)t.data + (size_t)column * dtype_size(t.dtype); }

class MLSTM : public Mixer {
public:
    MLSTM(const PartSpec& spec, BuildEnv&) {
        KeyReader r(spec.params, "mlstm", TQE_ERR_ARGUMENT);
        hidden_ = r.integer("hidden", 1);
        heads_ = (int)r.integer("heads", 1);
        d_ = (int)r.integer("head_dim", 1);
        dv_ = (int)r.integer("value_dim", 1);
        cap_ = (float)r.number("gate_cap", true);
        eps_ = (float)r.number("eps");
        q_scale_ = (float)r.number_or("q_scale", 1.0 / sqrt((double)d_));
        if (d_ > K::linear_attention_max_dim.raw()) raise(TQE_ERR_CONFIG, "mlstm: heads of %d key channels are more than the kernels take (%d)", d_, K::linear_attention_max_dim.raw());
        const Json& n = spec.params["names"];
        auto name = [&](const char* role, const char* fallback) { return n[role].is_string() ? n[role].as_string() : std::string(fallback); };
        n_q_ = name("q", "q"); n_k_ = name("k", "k"); n_v_ = name("v", "v"); n_g_ = name("g", "g"); n_o_ = name("o", "o"); n_norm_ = name("norm", "norm");
        n_i_ = name("i", "i"); n_ib_ = name("i_bias", "i.bias"); n_f_ = name("f", "f"); n_fb_ = name("f_bias", "f.bias");
        graph_safe = true;
    }
    TensorSpecs tensors() const override {
        auto w = [](int64_t a, int64_t b) { TensorSpec t; t.shape = {a, b}; return t; };
        auto bias = [](int64_t a, double std_dev) { TensorSpec t; t.shape = {a}; t.std_dev = std_dev; return t; };
        const int64_t qk = (int64_t)heads_ * d_, vv = (int64_t)heads_ * dv_;
        TensorSpec norm = bias(vv, 0.1);
        norm.init = "one_plus_normal";
        return {{n_q_, w(qk, hidden_)}, {n_k_, w(qk, hidden_)}, {n_v_, w(vv, hidden_)}, {n_g_, w(vv, hidden_)}, {n_o_, w(hidden_, vv)}, {n_norm_, norm},
                {n_i_, w(heads_, hidden_)}, {n_ib_, bias(heads_, 1.0)}, {n_f_, w(heads_, hidden_)}, {n_fb_, bias(heads_, 3.0)}};
    }
    void load(Loaded& t, hipStream_t stream) override {
        // (rows up to a multiple of 16, so that the products' rows stay at multiples of 16 bytes whatever the sizes)
        OwnedPtr in = stack_rows({take(t, n_q_), take(t, n_k_), take(t, n_v_), take(t, n_g_), take(t, n_i_), take(t, n_f_)}, stream, 16);
        row_ = in->t.shape[0];
        w_in_ = make_weight(in, 1, false, stream);
        // (the gates' rows a second time, for steps whose other rows are wanted in bfloat16)
        w_gates_ = make_weight(stack_rows({take(t, n_i_), take(t, n_f_)}, stream, 16), 1, false, stream);
        gate_bias_ = as_floats(stack_rows({take(t, n_ib_), take(t, n_fb_)}, stream), stream);
        w_o_ = make_weight(take(t, n_o_), 1, false, stream);
        norm_w_ = as_floats(take(t, n_norm_), stream);
        stored_ = t;
        for (const std::string& big : {n_q_, n_k_, n_v_, n_g_, n_o_}) stored_.erase(big);
    }
    OwnedPtr held(const std::string& name) const override {
        if (name == "in.weight") return w_in_.rows;
        if (name == "o.weight") return w_o_.rows;
        auto it = stored_.find(name);
        return it == stored_.end() ? nullptr : it->second;
    }
    const char* trace_name() const override { return "mlstm"; }
    void product_shapes(std::vector<std::pair<int64_t, int64_t>>& out) const override {
        out.push_back({(2LL * heads_ * d_ + 2LL * heads_ * dv_ + 2LL * heads_ + 15) / 16 * 16, hidden_});
        out.push_back({hidden_, (int64_t)heads_ * dv_});
    }
    CacheNeed cache_need() const override {
        CacheNeed n;
        n.kind = CacheNeed::State;
        n.state_shape = {(heads_ * head_stride() + heads_ + 3) / 4 * 4};
        n.state_dtype = F32;
        return n;
    }
    bool adds_to_stream(const StepContext& c) const override { return fusable(c.n_tokens, w_o_, true) || leaves_sums(c.n_tokens, w_o_); }

    Tensor forward(StepContext& c, const Activation& x, const CacheEntry& entry, Stream* stream, bool last_rows) override {
        if (!entry.state.defined() || !entry.writes) raise(TQE_ERR_STATE, "mlstm was given no state of its own in the cache");
        if (last_rows || x.lazy) raise(TQE_ERR_STATE, "mlstm takes all rows of the step, as they are");
        const int64_t n = x.x.shape[0];
        const int dtype = x.x.dtype;
        const long long row = entry.state.cols(), m_offset = heads_ * head_stride();
        float* state = (float*)entry.state.data + entry.state_offset;
        const int64_t qk = (int64_t)heads_ * d_, vv = (int64_t)heads_ * dv_;
        // many tokens in bfloat16 run in chunks on the matrix cores, whose operands are bfloat16; else one product gives everything in float32
        const bool chunked = dtype == BF16 && !c.all_decode && !c.capturing && c.max_new >= CHUNKED_FROM && !null_device() &&
                             K::mlstm_chunks_supported.raw(d_, dv_);
        const Tensor in = linear(c, x.x, w_in_, nullptr, chunked ? BF16 : F32).t;      // [q | k | v | g | i | f | padding]
        const Tensor z = chunked ? linear(c, x.x, w_gates_, nullptr, F32).t : Tensor();
        Tensor kappa = c.alloc(F32, {n, heads_}), tau = c.alloc(F32, {n, heads_}), m = c.alloc(F32, {n, heads_});
        Tensor gated = c.alloc(dtype, {n, vv});
        const float* norm_w = (const float*)norm_w_->t.data;
        const void* gate = at(in, 2 * qk + vv);
        Tensor o;
        if (chunked) {
            const Chunks ch = c.chunks(CHUNK);
            Tensor cs = c.alloc(F32, {ch.n, heads_, head_stride()}), cd = c.alloc(F32, {ch.n, heads_});
            const bool norms = K::mlstm_apply_norms.raw(dv_) != 0;
            if (!norms) o = c.alloc(F32, {n, heads_, dv_});
            K::mlstm_gate_scan((const float*)z.data, z.cols(), (const float*)gate_bias_->t.data, cap_, state, row, m_offset, c.dev.cu, c.dev.seq_new,
                               c.dev.seq_slot, (float*)kappa.data, (float*)tau.data, (float*)m.data, c.n_seqs, heads_, c.stream);
            K::mlstm_local(at(in, qk), at(in, 2 * qk), row_, (const float*)kappa.data, (const float*)tau.data, ch.row0, ch.count, ch.n, (float*)cs.data,
                           (float*)cd.data, heads_, d_, dv_, c.stream);
            K::chunk_carry((const float*)cd.data, heads_, (int)head_stride(), (float*)cs.data, ch.seq_first, c.dev.seq_slot, state, row, c.n_seqs, m_offset,
                           c.stream);
            K::mlstm_apply(in.data, at(in, qk), at(in, 2 * qk), row_, (const float*)kappa.data, (const float*)tau.data, (const float*)m.data, q_scale_, ch.row0,
                           ch.count, ch.n, (float*)cs.data, (float*)o.data, norm_w, eps_, gate, gated.data, heads_, d_, dv_, c.stream);
            if (!norms)
                K::head_norm_gate((const float*)o.data, norm_w, dv_, eps_, gate, dtype, row_, 1, gated.data, dtype, (int)n, heads_, dv_, c.stream);
            return finish(c, gated, stream);
        }
        Tensor inv_den = c.alloc(F32, {n, heads_});
        o = c.alloc(F32, {n, heads_, dv_});
        K::mlstm_gates((const float*)at(in, 2 * qk + 2 * vv), row_, (const float*)gate_bias_->t.data, cap_, in.data, at(in, qk), F32, row_, q_scale_, state, row,
                       head_stride(), m_offset, c.dev.cu, c.dev.seq_new, c.dev.seq_slot, (float*)kappa.data, (float*)tau.data, (float*)m.data,
                       (float*)inv_den.data, c.n_seqs, heads_, d_, c.stream);
        K::linear_attention(in.data, at(in, qk), at(in, 2 * qk), F32, row_, nullptr, 0, nullptr, 0.f, nullptr, (const float*)kappa.data,
                            (const float*)tau.data, (const float*)inv_den.data, nullptr, nullptr, q_scale_, 1.f, nullptr, nullptr, 0, 0, 0, c.dev.tok_pos, state, row, c.dev.cu,
                            c.dev.seq_new, c.dev.seq_slot, nullptr, nullptr, nullptr, nullptr, (float*)o.data, 0, c.n_seqs, heads_, d_, dv_, head_stride(),
                            c.stream);
        K::head_norm_gate((const float*)o.data, norm_w, dv_, eps_, gate, F32, row_, 1, gated.data, dtype, (int)n, heads_, dv_, c.stream);
        return finish(c, gated, stream);
    }

private:
    // steps that bring so many tokens of some sequence run in chunks on the matrix cores, shorter ones token by token
    static const int CHUNKED_FROM = 32, CHUNK = 64;

    Tensor finish(StepContext& c, const Tensor& gated, Stream* stream) {
        if (stream) {
            add_product(c, *stream, gated, w_o_);
            return Tensor();
        }
        return linear(c, gated, w_o_, nullptr, gated.dtype).t;
    }
    int64_t head_stride() const { return (int64_t)d_ * dv_ + d_; }

    int64_t hidden_, row_ = 0;
    int heads_, d_, dv_;
    float cap_ = 1.f, eps_ = 0.f, q_scale_ = 1.f;
    std::string n_q_, n_k_, n_v_, n_g_, n_o_, n_norm_, n_i_, n_ib_, n_f_, n_fb_;
    Weight w_in_, w_gates_, w_o_;
    OwnedPtr gate_bias_, norm_w_;
    Loaded stored_;
};

}  // namespace

void register_mlstm_parts() {
    register_kind("mixer", "mlstm", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<MLSTM>(s, e); });
}

}  // namespace tq
