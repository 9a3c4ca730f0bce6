// A mixer of time mixing: linear attention whose inputs each read a mix of their own of the token and the one before it, whose decay is a
// number per key channel and token, and whose current token is read through a bonus instead of the state.
//
//   time_mixing   with x' the previous token's x (zeros for a sequence's first), m_s = x + (x' - x) mu_s for s in r, k, v, g, w;
//                 r, k, v = W_r m_r, W_k m_k, W_v m_v (heads of head_dim elements), a = exp(-exp(W_w2 tanh(W_w1 m_w) + w0)) for all of
//                 their key channels; o_t = S_(t-1)^T r_t + (sum_i u_i k_i r_i) v_t, then S_t = diag(a_t) S_(t-1) + k_t v_t^T.  y = W_o (w_norm
//                 * [rms_norm(o) of every head] * silu(W_g m_g)), w_norm over all heads' elements.
//
// The cache's state row holds the state, [heads][head_dim][head_dim] float32, and behind it the last token's x (zero when a slot is taken).  The
// decay's second product, its exponentials, the recurrence and the heads' norm are float32 whatever the activation type; the other products are
// the framework's.  Steps that bring many tokens of a sequence run the recurrence in chunks: every chunk's own part of the state, a carry over the
// chunks, then the outputs; on the matrix cores where they take the heads' size (decay_chunks.hip).
//
// params: hidden, heads, head_dim, decay_rank (what random weights get: the checkpoint's tensors give the rank), eps, names {mu (a prefix: the mixes'
// weights are <mu>r, <mu>k, ...), r, k, v, g, o, w1, w2, w0, bonus, norm}.
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

// [a, b] float32 -> [b, a] (on the host, once)
OwnedPtr transposed(const OwnedPtr& p, hipStream_t stream) {
    const int64_t a = p->t.shape[0], b = p->t.shape[1];
    OwnedPtr out = make_owned(F32, {b, a});
    if (null_device()) return out;
    std::vector<float> in((size_t)(a * b)), turned(in.size());
    copy_to_host(in.data(), p->t.data, in.size() * 4, stream);
    for (int64_t i = 0; i < a; ++i)
        for (int64_t j = 0; j < b; ++j) turned[(size_t)(j * a + i)] = in[(size_t)(i * b + j)];
    copy_to_device(out->t.data, turned.data(), turned.size() * 4, stream);
    stream_synchronize(stream);
    return out;
}

class TimeMixing : public Mixer {
public:
    TimeMixing(const PartSpec& spec, BuildEnv&) {
        KeyReader r(spec.params, "time_mixing", TQE_ERR_ARGUMENT);
        hidden_ = r.integer("hidden", 1);
        heads_ = (int)r.integer("heads", 1);
        d_ = (int)r.integer("head_dim", 1);
        rank_ = r.integer_or("decay_rank", 16, 1);
        eps_ = (float)r.number("eps");
        if (d_ > K::linear_attention_max_dim.raw()) raise(TQE_ERR_CONFIG, "time_mixing: heads of %d key channels are more than the kernels take (%d)", d_, K::linear_attention_max_dim.raw());
        const Json& n = spec.params["names"];
        auto name = [&](const char* role, const char* fallback) { return n[role].is_string() ? n[role].as_string() : std::string(fallback); };
        n_mu_ = name("mu", "mu.");
        n_r_ = name("r", "r"); n_k_ = name("k", "k"); n_v_ = name("v", "v"); n_g_ = name("g", "g"); n_o_ = name("o", "o");
        n_w1_ = name("w1", "w1"); n_w2_ = name("w2", "w2"); n_w0_ = name("w0", "w0"); n_u_ = name("bonus", "u"); n_norm_ = name("norm", "norm");
        graph_safe = true;
    }
    TensorSpecs tensors() const override {
        auto w = [](int64_t a, int64_t b) { TensorSpec t; t.shape = {a, b}; return t; };
        auto v = [](int64_t a, double sd) { TensorSpec t; t.shape = {a}; t.std_dev = sd; return t; };
        const int64_t hd = (int64_t)heads_ * d_;
        TensorSpecs t;
        for (const char* s : MIXES) t.push_back({n_mu_ + s, v(hidden_, 0.3)});
        for (const std::string& p : {n_r_, n_k_, n_v_, n_g_}) t.push_back({p, w(hd, hidden_)});
        t.push_back({n_o_, w(hidden_, hd)});
        TensorSpec w1 = w(rank_, hidden_); w1.free = {0};
        TensorSpec w2 = w(hd, rank_); w2.free = {1}; w2.std_dev = 0.5;
        t.push_back({n_w1_, w1});
        t.push_back({n_w2_, w2});
        t.push_back({n_w0_, v(hd, 1.0)});
        t.push_back({n_u_, w(heads_, d_)});
        TensorSpec norm = v(hd, 0.1); norm.init = "one_plus_normal";
        t.push_back({n_norm_, norm});
        return t;
    }
    void load(Loaded& t, hipStream_t stream) override {
        std::vector<OwnedPtr> mu;
        for (const char* s : MIXES) mu.push_back(take(t, n_mu_ + s));
        OwnedPtr stacked = stack_rows(mu, stream);                       // [mixes * hidden]
        mu_ = as_floats(stacked, stream);
        const std::string* products[4] = {&n_r_, &n_k_, &n_v_, &n_g_};
        const int64_t hd = (int64_t)heads_ * d_;
        std::vector<OwnedPtr> four;
        for (int i = 0; i < 4; ++i) four.push_back(take(t, *products[i]));
        if (hd % 32 == 0) {
            // one behind the other, so that short steps run the four products in one launch
            w_all_ = make_weight(stack_rows(four, stream), 1, false, stream);
            for (int i = 0; i < 4; ++i) w_in_[i] = weight_slice(w_all_, i * hd, (i + 1) * hd);
        } else {
            for (int i = 0; i < 4; ++i) w_in_[i] = make_weight(four[(size_t)i], 1, false, stream);
        }
        w_o_ = make_weight(take(t, n_o_), 1, false, stream);
        OwnedPtr w1 = take(t, n_w1_), w2 = take(t, n_w2_);
        if (w1->t.shape[0] != w2->t.shape[1])
            raise(TQE_ERR_WEIGHTS, "time_mixing: the decay's two matrices do not meet: %s and %s", w1->t.describe().c_str(), w2->t.describe().c_str());
        rank_ = w1->t.shape[0];
        if (rank_ > K::low_rank_max.raw()) raise(TQE_ERR_WEIGHTS, "time_mixing: a decay of rank %lld is more than the kernel takes (%d)", (long long)rank_, K::low_rank_max.raw());
        w_w1_ = make_weight(w1, 1, false, stream);
        // (bfloat16 on the matrix cores takes the matrix as it is)
        on_cores_ = w2->t.dtype == BF16 && K::low_rank_mfma_supported.raw((int)rank_, (int)hd) != 0;
        if (on_cores_) w2_rows_ = w2;
        w2_ = transposed(as_floats(w2, stream), stream);
        w0_ = as_floats(take(t, n_w0_), stream);
        u_ = as_floats(take(t, n_u_), stream);
        norm_w_ = as_floats(take(t, n_norm_), stream);
        stored_ = t;
        for (const std::string& big : {n_r_, n_k_, n_v_, n_g_, n_o_, n_w1_, n_w2_}) stored_.erase(big);
    }
    OwnedPtr held(const std::string& name) const override {
        const std::string* products[4] = {&n_r_, &n_k_, &n_v_, &n_g_};
        for (int i = 0; i < 4; ++i)
            if (name == *products[i]) return w_in_[i].rows;
        if (name == n_o_) return w_o_.rows;
        auto it = stored_.find(name);
        return it == stored_.end() ? nullptr : it->second;
    }
    const char* trace_name() const override { return "linear-attn"; }
    void product_shapes(std::vector<std::pair<int64_t, int64_t>>& out) const override {
        out.push_back({(int64_t)heads_ * d_, hidden_});
        out.push_back({hidden_, (int64_t)heads_ * d_});
    }
    CacheNeed cache_need() const override {
        CacheNeed n;
        n.kind = CacheNeed::State;
        // (rows up to a multiple of four floats, so that every sequence's begins at 16 bytes)
        n.state_shape = {(last_at() + hidden_ + 3) / 4 * 4};
        n.state_dtype = F32;
        return n;
    }

    Tensor forward(StepContext& c, const Activation& x, const CacheEntry& entry, Stream* stream, bool last_rows) override {
        if (!entry.state.defined() || !entry.writes) raise(TQE_ERR_STATE, "time_mixing was given no state of its own in the cache");
        if (last_rows || x.lazy || stream) raise(TQE_ERR_STATE, "time_mixing takes all rows of the step, as they are, and returns its output");
        const int64_t n = x.x.shape[0], hd = (int64_t)heads_ * d_;
        const int dtype = x.x.dtype;
        const long long row = entry.state.cols();
        float* state = (float*)entry.state.data + entry.state_offset;
        float* last = state + last_at();
        // (the mixes one behind the other, each beginning at a multiple of 16 bytes)
        const int64_t mix_stride = (n * hidden_ + 7) / 8 * 8;
        const Tensor mixes = c.alloc(dtype, {N_MIXES, mix_stride});
        auto mix = [&](int i) { return Tensor((char*)mixes.data + (size_t)(i * mix_stride) * dtype_size(dtype), dtype, {n, hidden_}); };
        K::token_mixes(x.x.data, dtype, (const float*)mu_->t.data, N_MIXES, last, row, c.dev.tok_seq, c.dev.tok_pos, c.dev.seq_start, c.dev.seq_slot, mixes.data, mix_stride, (int)n,
                       (int)hidden_, c.all_decode ? 1 : 0, c.stream);
        if (!c.all_decode) K::rows_remember(x.x.data, dtype, last, row, c.dev.cu, c.dev.seq_new, c.dev.seq_slot, c.n_seqs, (int)hidden_, c.stream);
        // r, k, v, g: each a row of `stride` elements a token
        const void* part[4];
        long long stride = hd;
        if (dtype == BF16 && w_all_.defined() && takes_groups(n, w_all_, hd)) {
            const Tensor all = linear_groups(c, mix(0), mix_stride, w_all_, hd, dtype);
            stride = 4 * hd;
            for (int i = 0; i < 4; ++i) part[i] = (const char*)all.data + (size_t)(i * hd) * dtype_size(dtype);
        } else {
            for (int i = 0; i < 4; ++i) part[i] = linear(c, mix(i), w_in_[i], nullptr, dtype).t.data;
        }
        const Tensor low = linear(c, mix(4), w_w1_, nullptr, F32).t;
        Tensor log_decay = c.alloc(F32, {n, hd});
        const float* logs = (const float*)log_decay.data;
        if (dtype == BF16 && on_cores_)
            K::low_rank_decay_mfma((const float*)low.data, w2_rows_->t.data, (const float*)w0_->t.data, (float*)log_decay.data, (int)n, (int)rank_, (int)hd, c.stream);
        else
            K::low_rank_decay((const float*)low.data, (const float*)w2_->t.data, (const float*)w0_->t.data, (float*)log_decay.data, (int)n, (int)rank_, (int)hd, c.stream);
        const float* u = (const float*)u_->t.data;
        const float* norm_w = (const float*)norm_w_->t.data;
        Tensor gated = c.alloc(dtype, {n, hd});
        const bool many = dtype == BF16 && !c.all_decode && !c.capturing && !null_device();
        if (many && c.max_new >= CORES_FROM && K::decay_chunks_supported.raw(d_, d_)) {
            // on the matrix cores, the heads' norm and the gate in the last kernel
            const Chunks ch = c.chunks(CHUNK);
            Tensor cs = c.alloc(F32, {ch.n, hd * d_}), cd = c.alloc(F32, {ch.n, hd});
            K::decay_local(part[1], part[2], stride, logs, ch.row0, ch.count, ch.n, (float*)cs.data, (float*)cd.data, heads_, d_, d_, c.stream);
            K::chunk_carry((const float*)cd.data, hd, d_, (float*)cs.data, ch.seq_first, c.dev.seq_slot, state, row, c.n_seqs, hd * d_, c.stream);
            K::decay_apply(part[0], part[1], part[2], stride, logs, u, ch.row0, ch.count, ch.n, (float*)cs.data, norm_w, eps_, part[3], stride, gated.data,
                           heads_, d_, d_, c.stream);
            return linear(c, gated, w_o_, nullptr, dtype).t;
        }
        Tensor o = c.alloc(F32, {n, heads_, d_});
        auto run = [&](int mode, int items, const Chunks* ch, float* cs, float* cd) {
            K::linear_attention(part[0], part[1], part[2], dtype, stride, nullptr, 0, nullptr, 0.f, nullptr, nullptr, nullptr, nullptr, logs, u, 1.f, 1.f, nullptr,
                                nullptr, 0, 0, 0, c.dev.tok_pos, state, row, c.dev.cu, c.dev.seq_new, c.dev.seq_slot, ch ? ch->row0 : nullptr, ch ? ch->count : nullptr,
                                cs, cd, (float*)o.data, mode, items, heads_, d_, d_, (long long)d_ * d_, c.stream);
        };
        if (many && c.max_new >= CHUNKED_FROM) {
            const Chunks ch = c.chunks(CHUNK);
            Tensor cs = c.alloc(F32, {ch.n, hd * d_}), cd = c.alloc(F32, {ch.n, hd});
            run(1, ch.n, &ch, (float*)cs.data, (float*)cd.data);
            K::chunk_carry((const float*)cd.data, hd, d_, (float*)cs.data, ch.seq_first, c.dev.seq_slot, state, row, c.n_seqs, hd * d_, c.stream);
            run(2, ch.n, &ch, (float*)cs.data, (float*)cd.data);
        } else {
            run(0, c.n_seqs, nullptr, nullptr, nullptr);
        }
        K::head_norm_gate((const float*)o.data, norm_w, d_, eps_, part[3], dtype, stride, 0, gated.data, dtype, (int)n, heads_, d_, c.stream);
        return linear(c, gated, w_o_, nullptr, dtype).t;
    }

private:
    // steps that bring so many tokens of some sequence run in chunks: on the matrix cores, or (sizes those do not take) on the vector units
    static const int CORES_FROM = 32, CHUNKED_FROM = 128, CHUNK = 64, N_MIXES = 5;
    static constexpr const char* MIXES[N_MIXES] = {"r", "k", "v", "g", "w"};
    // where a state row keeps the last token's x: behind the state, at a multiple of four floats
    int64_t last_at() const { return ((int64_t)heads_ * d_ * d_ + 3) / 4 * 4; }
    int64_t hidden_, rank_;
    int heads_, d_;
    float eps_;
    std::string n_mu_, n_r_, n_k_, n_v_, n_g_, n_o_, n_w1_, n_w2_, n_w0_, n_u_, n_norm_;
    Weight w_all_, w_in_[4], w_o_, w_w1_;      // the four products stacked (or not defined); each of them
    OwnedPtr mu_, w2_, w2_rows_, w0_, u_, norm_w_;      // w2_: [rank, channels] float32; w2_rows_: as the checkpoint has it
    bool on_cores_ = false;
    Loaded stored_;
};
constexpr const char* TimeMixing::MIXES[];

}  // namespace

void register_time_mixing_parts() {
    register_kind("mixer", "time_mixing", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<TimeMixing>(s, e); });
}

}  // namespace tq
