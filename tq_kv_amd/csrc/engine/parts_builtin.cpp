// The built-in kinds: RMSNorm, rotary positions (and none), grouped-query softmax attention,
// the gated-SiLU feed-forward, and the pre-norm block arrangement.
#include <math.h>

#include <mutex>

#include "kernels.h"
#include "linear.h"
#include "parts.h"
#include "step.h"
#include "trace.h"

namespace tq {

// ---- registry ----------------------------------------------------------------------------------
namespace {
const char* const CATEGORIES[] = {"norm", "position", "mixer", "feed_forward", "block"};
std::map<std::string, std::map<std::string, Factory>>& registry() {
    static std::map<std::string, std::map<std::string, Factory>> r;
    return r;
}
std::mutex g_registry_mutex;

std::string joined(const std::vector<std::string>& v) {
    std::string s;
    for (size_t i = 0; i < v.size(); ++i) s += (i ? ", " : "") + v[i];
    return s;
}
}  // namespace

void register_kind(const std::string& category, const std::string& kind, Factory factory) {
    bool known = false;
    for (const char* c : CATEGORIES) known = known || category == c;
    if (!known) raise(TQE_ERR_ARGUMENT, "unknown part category '%s' (known: norm, position, mixer, feed_forward, block)", category.c_str());
    std::lock_guard<std::mutex> lock(g_registry_mutex);
    registry()[category][kind] = std::move(factory);
}

std::vector<std::string> known_kinds(const std::string& category) {
    register_builtin_parts();
    std::lock_guard<std::mutex> lock(g_registry_mutex);
    std::vector<std::string> out;
    for (const auto& e : registry()[category]) out.push_back(e.first);
    return out;
}

std::shared_ptr<Part> build_part(const std::string& category, const PartSpec& spec, BuildEnv& env) {
    register_builtin_parts();
    Factory f;
    {
        std::lock_guard<std::mutex> lock(g_registry_mutex);
        auto& kinds = registry()[category];
        auto it = kinds.find(spec.kind);
        if (it != kinds.end()) f = it->second;
    }
    if (!f) raise(TQE_ERR_ARGUMENT, "unknown %s kind '%s' (known: %s)", category.c_str(), spec.kind.c_str(), joined(known_kinds(category)).c_str());
    std::shared_ptr<Part> p = f(spec, env);
    p->category = category;
    p->kind = spec.kind;
    return p;
}

Json Part::describe() const {
    Json j = Json::object();
    j.set("category", category);
    j.set("kind", kind);
    j.set("graph_safe", graph_safe);
    Json ts = Json::object();
    for (const auto& t : tensors()) ts.set(t.first, t.second.to_json());
    j.set("tensors", ts);
    return j;
}

bool Norm::lazy(const Stream& stream, LazyNorm& out) const {
    if (stream.pending.kind != Pending::Nothing || stream.xw_for != this) return false;
    out.xw = stream.xw_buffer;
    out.ss = stream.ss_buffer;
    out.n_ss = stream.n_ss;
    out.eps = fold_eps();
    return true;
}

static OwnedPtr take(Loaded& tensors, const char* name) {
    auto it = tensors.find(name);
    if (it == tensors.end() || !it->second) raise(TQE_ERR_WEIGHTS, "a part was not given its tensor '%s'", name);
    return it->second;
}

static OwnedPtr as_floats(const OwnedPtr& p, hipStream_t stream) {
    if (p->t.dtype == F32) return p;
    std::vector<int64_t> dims(p->t.shape, p->t.shape + p->t.ndim);
    OwnedPtr out = make_owned(F32, dims);
    if (!null_device()) K::convert(p->t.data, p->t.dtype, out->t.data, F32, (long long)p->t.numel(), stream);
    stream_synchronize(stream);
    return out;
}

// ---- RMSNorm -----------------------------------------------------------------------------------
// As the reference computes it (src/models/turbo_generic.rs:41-51): x / sqrt(mean(x^2) + eps) *
// weight in float32, cast last; the weight is used as it is stored (no 1 + w).
//
// params: size, eps; optional unit_offset (true: the stored weight lies around zero and the norm multiplies by
// 1 + w; the sum is formed once, in float32, when the weight is loaded) and tensor (the name of the weight inside
// the part's prefix, "weight" unless given; it may be empty where the prefix is the whole name).
class RMSNorm : public Norm {
public:
    RMSNorm(const PartSpec& spec, BuildEnv& env) : act_dtype_(env.act_dtype) {
        KeyReader r(spec.params, "rms_norm", TQE_ERR_ARGUMENT);
        size_ = r.integer("size", 1);
        eps_ = (float)r.number("eps");
        unit_offset_ = r.boolean_or("unit_offset", false);
        tensor_ = r.string_or("tensor", "weight");
        graph_safe = true;
    }
    TensorSpecs tensors() const override {
        TensorSpec t;
        t.shape = {size_};
        t.init = unit_offset_ ? "normal" : "one_plus_normal";
        if (unit_offset_) t.std_dev = 0.1;
        return {{tensor_, t}};
    }
    void load(Loaded& tensors, hipStream_t stream) override {
        stored_ = take(tensors, tensor_.c_str());
        weight_ = stored_;
        if (!unit_offset_) return;
        // 1 + w in float32, made on the host (a vector of the model's width, once)
        const Tensor& t = stored_->t;
        std::vector<float> host((size_t)t.numel());
        if (t.dtype == F32) copy_to_host(host.data(), t.data, t.bytes(), stream);
        else {
            std::vector<uint16_t> bits((size_t)t.numel());
            copy_to_host(bits.data(), t.data, t.bytes(), stream);
            for (size_t i = 0; i < bits.size(); ++i) {
                const uint32_t u = (uint32_t)bits[i] << 16;
                memcpy(&host[i], &u, 4);
            }
        }
        for (float& v : host) v = 1.0f + v;
        weight_ = make_owned(F32, {size_});
        copy_to_device(weight_->t.data, host.data(), host.size() * 4, stream);
        stream_synchronize(stream);
    }
    OwnedPtr held(const std::string& name) const override { return name == tensor_ ? stored_ : name == "weight.effective" ? weight_ : nullptr; }
    const char* trace_name() const override { return "rms-norm"; }          // the reference's span, src/models/turbo_generic.rs:36
    int64_t size() const override { return size_; }

    void forward(StepContext& c, const Tensor& x, Tensor& out) override {
        k_add_rmsnorm(c, nullptr, Pending::of(x), weight_->t, eps_, nullptr, out.shape[0], x.shape[0], out, false);
    }
    void add_norm(StepContext& c, Tensor& h, const Pending& delta, Tensor& out) override {
        k_add_rmsnorm(c, (float*)h.data, delta, weight_->t, eps_, nullptr, out.shape[0], h.shape[0], out, delta.kind != Pending::Nothing);
    }
    void gather_add_norm(StepContext& c, const Tensor& h, const Pending& delta, const int32_t* rows, int64_t n_rows, Tensor& out) override {
        k_add_rmsnorm(c, (float*)h.data, delta, weight_->t, eps_, rows, n_rows, h.shape[0], out, false);
    }
    bool takes_partial_sums() const override { return true; }
    // (the weight as stored, bfloat16, or the sum 1 + w, float32: the kernels that prepare a norm take either)
    bool foldable() const override { return weight_ && (weight_->t.dtype == BF16 || (unit_offset_ && weight_->t.dtype == F32)); }
    const Tensor* fold_weight() const override { return &weight_->t; }
    float fold_eps() const override { return eps_; }

private:
    int64_t size_;
    float eps_;
    int act_dtype_;
    bool unit_offset_;
    std::string tensor_;
    OwnedPtr stored_, weight_;       // what the checkpoint holds; what the kernels multiply by
};

// ---- positions ---------------------------------------------------------------------------------
// Rotary tables as the reference builds them (src/models/turbo_generic.rs:1654-1670): theta_j =
// 1 / base^(2j/d) with base rounded to float32 and the power taken in float32, angle = position *
// theta_j in float32, cos and sin of it.  Layouts: halves (:417-427, what Qwen2 uses) and pairs
// (:430-443); rot_dim < head_dim rotates the first rot_dim elements only (:752-761).
//
// Optional scaling {factor, low, high, original}: a frequency f with wavelength l = 2 pi / f stays as it is where l < original / high, becomes
// f / factor where l > original / low, and between the two (1 - s) f / factor + s f with s = (original / l - low) / (high - low).
class Rotary : public Position {
public:
    Rotary(const PartSpec& spec, BuildEnv&) {
        KeyReader r(spec.params, "rotary", TQE_ERR_ARGUMENT);
        theta_ = r.number("theta");
        rot_dim_ = (int)r.integer("rot_dim");
        max_positions = r.integer("max_positions", 1);
        const std::string style = r.string_or("style", "halves");
        if (style == "halves") style_ = STYLE_HALVES;
        else if (style == "pairs") style_ = STYLE_PAIRS;
        else raise(TQE_ERR_ARGUMENT, "rotary: unknown style '%s' (known: halves, pairs)", style.c_str());
        if (rot_dim_ <= 0 || rot_dim_ % 2) raise(TQE_ERR_ARGUMENT, "rotary: rot_dim must be even and positive, got %d", rot_dim_);
        graph_safe = true;
        // The tables are computed on the host in float32, so that they are the same numbers
        // whatever device the model runs on.
        const int half = rot_dim_ / 2;
        std::vector<float> cos_h((size_t)max_positions * half), sin_h(cos_h.size());
        const float base = (float)theta_;
        std::vector<float> inv((size_t)half);
        for (int j = 0; j < half; ++j) inv[(size_t)j] = 1.0f / powf(base, (float)(2 * j) / (float)rot_dim_);
        if (!spec.params["scaling"].is_null()) {
            KeyReader sc(spec.params["scaling"], "rotary: scaling", TQE_ERR_ARGUMENT);
            const double factor = sc.number("factor", true), low = sc.number("low", true), high = sc.number("high", true), original = sc.number("original", true);
            for (float& f : inv) {
                const double length = 2.0 * M_PI / (double)f;
                if (length < original / high) continue;
                if (length > original / low) { f = (float)((double)f / factor); continue; }
                const double s = (original / length - low) / (high - low);
                f = (float)((1.0 - s) * (double)f / factor + s * (double)f);
            }
        }
        for (int64_t p = 0; p < max_positions; ++p)
            for (int j = 0; j < half; ++j) {
                const float angle = (float)p * inv[(size_t)j];
                cos_h[(size_t)p * half + j] = cosf(angle);
                sin_h[(size_t)p * half + j] = sinf(angle);
            }
        cos_ = make_owned(F32, {max_positions, half});
        sin_ = make_owned(F32, {max_positions, half});
        copy_to_device(cos_->t.data, cos_h.data(), cos_h.size() * 4, nullptr);
        copy_to_device(sin_->t.data, sin_h.data(), sin_h.size() * 4, nullptr);
        stream_synchronize(nullptr);
    }
    Tables tables() const override {
        Tables t;
        t.cos = cos_->t;
        t.sin = sin_->t;
        t.rot_dim = rot_dim_;
        t.style = style_;
        return t;
    }
    OwnedPtr held(const std::string& name) const override { return name == "cos" ? cos_ : name == "sin" ? sin_ : nullptr; }

private:
    double theta_;
    int rot_dim_, style_;
    OwnedPtr cos_, sin_;
};

// No change of q and k (a mixer that needs no positions, or learns them elsewhere).
class NoPosition : public Position {
public:
    NoPosition(const PartSpec& spec, BuildEnv&) {
        KeyReader r(spec.params, "position none", TQE_ERR_ARGUMENT);
        max_positions = r.integer_or("max_positions", (long long)1 << 30, 1);
        graph_safe = true;
    }
};

// ---- attention -----------------------------------------------------------------------------------
// Grouped-query softmax attention over the cache.  Order of work as in the reference
// (src/models/turbo_generic.rs:770-833, 1604-1635): q, k, v projections (+ bias), head split,
// position encoding of q and k, keys and values into the cache, scores q.k/sqrt(d), mask, softmax,
// p.v, merge heads, output projection without bias.  Query head h reads kv head h // (heads //
// kv_heads) (:195-204).  The three projections are one product with the weights stacked.
//
// params: hidden, n_heads, n_kv_heads, head_dim, qkv_bias, out_bias, window (null or positions a
// query sees, itself included), scale (null: 1/sqrt(head_dim)), position (a part spec); optional
// prompt_tile: queries per tile of the prompt kernel (16, 32, 64 or 128).
//
// What other designs put around the same attention, all off unless given: value_dim (a head's values are of another
// size than its keys); values_are_keys (there is no value projection: the values are the keys as projected, before norm and rotation);
// qk_norm with eps (every query and key head is divided by its root mean square and multiplied
// by a weight of head_dim values, before the rotation; with qk_norm_weight false and qk_norm_after_rotation true the heads are divided by
// their root mean square after the rotation and there is no weight); cap (scores become cap tanh(s / cap)); chunk (positions fall into
// chunks of so many, counted from the sequence's start, and see nothing of an earlier chunk); keep_first (with a
// window: a sequence's first positions stay visible, at their true places); sink (a learned number per head whose
// exponential joins the softmax's denominator, with no key and no value); value_mix "source" (the values of the
// step's tokens are handed to later layers) or "mixed" (v <- (1 - lambda) v + lambda v_source with a learned scalar,
// before the cache); value_mix_key (which source, "values" unless given); cache_keeps_all (the cache keeps every page although the
// mixer sees a window); cache_window (the cache keeps so many positions although the mixer sees a smaller window: another run reads them);
// qk_norm_over "projection" (with qk_norm: all of q, and all of k, are divided by the root mean square of the whole projection and multiplied by a
// weight of its size, before the rotation); sink_score (a number: a sink of that fixed score for every head, without a tensor); gate "head" (a
// head's output is multiplied by the sigmoid of a product of its own with the mixer's input); own_kv false (no projections of keys and
// values: the run reads another run's cache); names: the tensors' names inside the
// part's prefix {q, k, v, o, q_norm, k_norm, sink, mix, gate}.  With any of them the step runs through the kernels of
// attention_masked.hip.
//
// Its pages: keys [kv heads, page, head_dim]; values [kv heads, head_dim, page], transposed inside
// a page and the page's positions in the order the matrix cores take them (the kernels' own
// layout, which is why the mixer names the shapes and the cache only multiplies them out).
class Attention : public Mixer {
public:
    static const int DECODE_KERNEL_ROWS = 32;       // up to so many rows of a prompt step go through the decoding kernel

    Attention(const PartSpec& spec, BuildEnv& env) : act_dtype_(env.act_dtype) {
        KeyReader r(spec.params, "attention", TQE_ERR_ARGUMENT);
        hidden_ = r.integer("hidden", 1);
        n_heads_ = (int)r.integer("n_heads", 1);
        n_kv_heads_ = (int)r.integer("n_kv_heads", 1);
        head_dim_ = (int)r.integer("head_dim", 1);
        qkv_bias_ = r.boolean_or("qkv_bias", false);
        out_bias_ = r.boolean_or("out_bias", false);
        window_ = r.has("window") ? (int)r.integer("window") : 0;
        if (n_heads_ % n_kv_heads_) raise(TQE_ERR_ARGUMENT, "attention: %d heads are not a multiple of %d kv heads", n_heads_, n_kv_heads_);
        if (r.has("window") && window_ < 1) raise(TQE_ERR_ARGUMENT, "attention: window must be at least 1, got %d", window_);
        scale_ = r.has("scale") ? (float)r.number("scale") : (float)(1.0 / sqrt((double)head_dim_));
        prompt_tile_ = r.has("prompt_tile") ? (int)r.integer("prompt_tile") : 0;
        value_dim_ = r.has("value_dim") ? (int)r.integer("value_dim", 1) : head_dim_;
        qk_norm_ = r.boolean_or("qk_norm", false);
        qk_norm_weight_ = r.boolean_or("qk_norm_weight", true);
        norm_after_rotation_ = r.boolean_or("qk_norm_after_rotation", false);
        eps_ = qk_norm_ ? (float)r.number("eps") : 0.f;
        values_are_keys_ = r.boolean_or("values_are_keys", false);
        if (values_are_keys_ && value_dim_ != head_dim_)
            raise(TQE_ERR_ARGUMENT, "attention: keys of %d elements cannot serve as values of %d", head_dim_, value_dim_);
        chunk_ = r.has("chunk") ? (int)r.integer("chunk", 1) : 0;
        cap_ = r.has("cap") ? (float)r.number("cap", true) : 0.f;
        keep_first_ = (int)r.integer_or("keep_first", 0, 0);
        cache_keeps_all_ = r.boolean_or("cache_keeps_all", false);
        has_sink_ = r.boolean_or("sink", false);
        fixed_sink_ = r.has("sink_score");
        if (fixed_sink_) sink_score_ = (float)r.number("sink_score");
        if (has_sink_ && fixed_sink_) raise(TQE_ERR_ARGUMENT, "attention: a learned sink and one of a fixed score");
        const std::string norm_over = r.string_or("qk_norm_over", "head");
        if (norm_over != "head" && norm_over != "projection") raise(TQE_ERR_ARGUMENT, "attention: unknown qk_norm_over '%s' (known: head, projection)", norm_over.c_str());
        const std::string gate = r.string_or("gate", "none");
        if (gate != "none" && gate != "head") raise(TQE_ERR_ARGUMENT, "attention: unknown gate '%s' (known: none, head)", gate.c_str());
        gated_ = gate == "head";
        own_kv_ = r.boolean_or("own_kv", true);
        cache_window_ = r.has("cache_window") ? (int)r.integer("cache_window", 1) : window_;
        if (cache_window_ < window_ || (window_ == 0 && cache_window_ != 0)) raise(TQE_ERR_ARGUMENT, "attention: the cache keeps %d positions, the mixer sees %d", cache_window_, window_);
        // one kernel puts a norm over the projection, a gate per head and queries alone between the product and the attention
        projected_ = (qk_norm_ && norm_over == "projection") || gated_ || !own_kv_;
        const std::string mixing = r.string_or("value_mix", "none");
        if (mixing == "none") value_mix_ = MIX_NONE;
        else if (mixing == "source") value_mix_ = MIX_SOURCE;
        else if (mixing == "mixed") value_mix_ = MIX_MIXED;
        else raise(TQE_ERR_ARGUMENT, "attention: unknown value_mix '%s' (known: none, source, mixed)", mixing.c_str());
        mix_key_ = "attention." + r.string_or("value_mix_key", "values");
        if (keep_first_ > 0 && window_ == 0) raise(TQE_ERR_ARGUMENT, "attention: keep_first %d without a window", keep_first_);
        extras_ = value_dim_ != head_dim_ || values_are_keys_ || chunk_ > 0 || qk_norm_ || cap_ > 0.f || keep_first_ > 0 || has_sink_ || fixed_sink_ || projected_ ||
                  value_mix_ != MIX_NONE;
        if (projected_ && (values_are_keys_ || value_mix_ != MIX_NONE || (qk_norm_ && (norm_over != "projection" || !qk_norm_weight_ || norm_after_rotation_))))
            raise(TQE_ERR_ARGUMENT, "attention: a gate, a norm over the projection or borrowed keys and values go with values of their own that are not mixed, and no norm of heads");
        if (qk_norm_ && qk_norm_weight_ == norm_after_rotation_)
            raise(TQE_ERR_ARGUMENT, "attention: the heads' norm is either weighted and in front of the rotation, or without a weight and after it");
        // the kernel that adds biases, turns and then norms without a weight stands for every such combination but mixed values and
        // values that are the keys; the one that norms in front of the rotation for every other
        const bool turned_ok = extras_ && !projected_ && (!qk_norm_ || norm_after_rotation_) && value_mix_ == MIX_NONE && !values_are_keys_;
        if (extras_ && norm_after_rotation_ && qk_norm_ && !turned_ok)
            raise(TQE_ERR_ARGUMENT, "attention: a heads' norm after the rotation goes with values of their own that are not mixed");
        if (extras_ && out_bias_)
            raise(TQE_ERR_ARGUMENT, "attention: with value_dim, values_are_keys, chunk, qk_norm, cap, keep_first, sink or value_mix the output has no bias");
        {
            const Json& names = spec.params["names"];
            auto name = [&](const char* role, const char* fallback) { return names[role].is_string() ? names[role].as_string() : std::string(fallback); };
            n_q_ = name("q", "q_proj.weight"); n_k_ = name("k", "k_proj.weight"); n_v_ = name("v", "v_proj.weight"); n_o_ = name("o", "o_proj.weight");
            n_q_norm_ = name("q_norm", "q_norm.weight"); n_k_norm_ = name("k_norm", "k_norm.weight");
            n_sink_ = name("sink", "sink"); n_mix_ = name("mix", "value_mix"); n_gate_ = name("gate", "gate.weight");
            n_qb_ = name("q_bias", "q_proj.bias"); n_kb_ = name("k_bias", "k_proj.bias"); n_vb_ = name("v_bias", "v_proj.bias");
        }
        if (r.has("prompt_tile") && prompt_tile_ != 16 && prompt_tile_ != 32 && prompt_tile_ != 64 && prompt_tile_ != 128)
            raise(TQE_ERR_ARGUMENT, "attention: prompt_tile must be 16, 32, 64 or 128, got %d", prompt_tile_);
        // what no attention kernel takes is refused here, before any weight is read
        const int max_d = K::attention_max_head_dim.raw();
        if (head_dim_ > max_d)
            raise(TQE_ERR_CONFIG, "attention: head_dim %d is more than the attention kernels take (%d)", head_dim_, max_d);
        if (n_heads_ > 65535) raise(TQE_ERR_CONFIG, "attention: %d heads are more than the attention kernels take (65535)", n_heads_);
        if (extras_ && std::max(head_dim_, value_dim_) > K::attention_masked_max_dim.raw())
            raise(TQE_ERR_CONFIG, "attention: heads of %d and %d values are more than the attention kernels take (%d)", head_dim_, value_dim_,
                  K::attention_masked_max_dim.raw());
        const PartSpec pos = PartSpec::from_json(spec.params["position"], "attention: position");
        const std::string key = "position:" + pos.key();
        auto it = env.shared.find(key);
        if (it == env.shared.end()) it = env.shared.emplace(key, build_part("position", pos, env)).first;
        position_ = std::dynamic_pointer_cast<Position>(it->second);
        if (!position_) raise(TQE_ERR_ARGUMENT, "attention: part kind '%s' is no position", pos.kind.c_str());
        graph_safe = !position_->has_apply() || position_->graph_safe;
        takes_rows = true;
        if (extras_) {
            const Position::Tables tb = position_->tables();
            turned_first_ = turned_ok && (qkv_bias_ || norm_after_rotation_ || tb.style == STYLE_PAIRS);
            if (position_->has_apply() || tb.rot_dim > head_dim_)
                raise(TQE_ERR_ARGUMENT, "attention: with value_dim, values_are_keys, chunk, qk_norm, cap, keep_first, sink or value_mix the position part must turn from tables");
        }
    }

    TensorSpecs tensors() const override {
        const int64_t q = (int64_t)n_heads_ * head_dim_, kv = (int64_t)n_kv_heads_ * head_dim_;
        auto w = [](int64_t a, int64_t b) { TensorSpec t; t.shape = {a, b}; return t; };
        auto b = [](int64_t a) { TensorSpec t; t.shape = {a}; return t; };
        TensorSpecs t = {{n_q_, w(q, hidden_)}};
        if (own_kv_) t.push_back({n_k_, w(kv, hidden_)});
        if (own_kv_ && !values_are_keys_) t.push_back({n_v_, w((int64_t)n_kv_heads_ * value_dim_, hidden_)});
        if (gated_) t.push_back({n_gate_, w(n_heads_, hidden_)});
        t.push_back({n_o_, w(hidden_, (int64_t)n_heads_ * value_dim_)});
        if (qk_norm_ && qk_norm_weight_) {
            TensorSpec n = b(projected_ ? q : head_dim_);
            n.init = "one_plus_normal";
            n.std_dev = 0.1;
            t.push_back({n_q_norm_, n});
            n.shape = {projected_ ? kv : head_dim_};
            if (own_kv_) t.push_back({n_k_norm_, n});
        }
        if (has_sink_) { TensorSpec s = b(n_heads_); s.std_dev = 1.0; t.push_back({n_sink_, s}); }
        // the source layer of a mix has the scalar too, and does not use it
        if (value_mix_ != MIX_NONE) { TensorSpec s; s.shape = {}; s.std_dev = 0.3; t.push_back({n_mix_, s}); }
        if (qkv_bias_) {
            t.push_back({n_qb_, b(q)});
            if (own_kv_) t.push_back({n_kb_, b(kv)});
            if (own_kv_ && !values_are_keys_) t.push_back({n_vb_, b((int64_t)n_kv_heads_ * value_dim_)});
        }
        if (out_bias_) t.push_back({"o_proj.bias", b(hidden_)});
        return t;
    }

    void load(Loaded& t, hipStream_t stream) override {
        auto stack_of = [&](const std::string& q, const std::string& k, const std::string& v) {
            std::vector<OwnedPtr> parts = {take(t, q.c_str())};
            if (own_kv_) parts.push_back(take(t, k.c_str()));
            if (own_kv_ && !values_are_keys_) parts.push_back(take(t, v.c_str()));
            return parts;
        };
        std::vector<OwnedPtr> first = stack_of(n_q_, n_k_, n_v_);
        if (gated_) first.push_back(take(t, n_gate_.c_str()));
        // (rows up to a multiple of 16 where the gate's stand behind the others, so that the product's rows stay at multiples of 16 bytes)
        OwnedPtr qkv = stack_rows(first, stream, projected_ ? 16 : 1);
        row_ = qkv->t.shape[0];
        if (qk_norm_ && qk_norm_weight_) { q_norm_ = take(t, n_q_norm_.c_str()); if (own_kv_) k_norm_ = take(t, n_k_norm_.c_str()); }
        if (has_sink_) sink_ = take(t, n_sink_.c_str());
        if (fixed_sink_) {
            const std::vector<float> scores((size_t)n_heads_, sink_score_);
            sink_ = make_owned(F32, {n_heads_});
            copy_to_device(sink_->t.data, scores.data(), scores.size() * 4, stream);
            stream_synchronize(stream);
        }
        if (value_mix_ != MIX_NONE) mix_ = take(t, n_mix_.c_str());
        if (qkv_bias_) b_qkv_ = stack_rows(stack_of(n_qb_, n_kb_, n_vb_), stream);
        if (projected_) {
            // (small vectors, read in float32 by the kernel behind the product)
            if (b_qkv_) bias_f_ = as_floats(b_qkv_, stream);
            if (q_norm_) q_norm_f_ = as_floats(q_norm_, stream);
            if (k_norm_) k_norm_f_ = as_floats(k_norm_, stream);
        }
        if (out_bias_) b_o_ = take(t, "o_proj.bias");
        w_qkv_ = make_weight(qkv, 1, false, stream);
        w_o_ = make_weight(take(t, n_o_.c_str()), 1, b_o_ != nullptr, stream);
    }
    OwnedPtr held(const std::string& name) const override {
        if (name == "qkv.weight") return w_qkv_.rows;
        if (name == "qkv.weight.packed") return w_qkv_.packed;
        if (name == "qkv.bias") return b_qkv_;
        if (name == "o_proj.weight") return w_o_.rows;
        if (name == "o_proj.weight.packed") return w_o_.packed;
        if (q_norm_ && name == n_q_norm_) return q_norm_;
        if (k_norm_ && name == n_k_norm_) return k_norm_;
        if (has_sink_ && name == n_sink_) return sink_;
        if (name == "sink.score") return fixed_sink_ ? sink_ : nullptr;
        if (value_mix_ != MIX_NONE && name == n_mix_) return mix_;
        return nullptr;
    }
    const char* trace_name() const override { return "attn"; }             // the reference's span, src/models/turbo_generic.rs:1920
    void product_shapes(std::vector<std::pair<int64_t, int64_t>>& out) const override {
        int64_t n = (int64_t)n_heads_ * head_dim_ + (gated_ ? n_heads_ : 0);
        if (own_kv_) n += (int64_t)n_kv_heads_ * head_dim_ + (values_are_keys_ ? 0 : (int64_t)n_kv_heads_ * value_dim_);
        out.push_back({projected_ ? (n + 15) / 16 * 16 : n, hidden_});
        out.push_back({hidden_, (int64_t)n_heads_ * value_dim_});
    }

    CacheNeed cache_need() const override {
        CacheNeed n;
        n.kind = CacheNeed::Pages;
        n.key_page = {n_kv_heads_, TQE_PAGE, head_dim_};
        n.value_page = {n_kv_heads_, value_dim_, TQE_PAGE};
        // (cache_keeps_all: the cache gives no page back although the mixer sees a window, so that layers of many different windows
        // can share one group of the cache)
        n.window = cache_keeps_all_ ? 0 : cache_window_;
        n.keep_first = cache_keeps_all_ ? 0 : keep_first_;
        n.chunk = cache_keeps_all_ ? 0 : chunk_;
        return n;
    }

    // The folded q/k/v kernel takes decoding steps (row m is sequence m) of rotary positions in the
    // halves layout over the whole head.
    bool fused_qkv_ok(const StepContext& c) const {
        if (extras_ || !(c.all_decode && fusable(c.n_tokens, w_qkv_) && head_dim_ % 32 == 0)) return false;
        if (position_->has_apply()) return false;
        const Position::Tables tb = position_->tables();
        if (tb.style != STYLE_HALVES || tb.rot_dim != head_dim_) return false;
        return !b_qkv_ || b_qkv_->t.dtype == BF16;
    }
    bool folds_norm(const StepContext& c) const override {
        // (with biases first and the heads' norm after the rotation: the product alone divides by the rows' root mean square)
        if (extras_) return turned_first_ && c.all_decode && fusable(c.n_tokens, w_qkv_) && !reads_other_cache;
        return fused_qkv_ok(c) && !reads_other_cache;
    }
    bool adds_to_stream(const StepContext& c) const override {
        return !b_o_ && (fusable(c.n_tokens, w_o_, true) || leaves_sums(c.n_tokens, w_o_));
    }

    Tensor forward(StepContext& c, const Activation& x, const CacheEntry& entry, Stream* stream, bool last_rows) override {
        if (entry.kind != CacheNeed::Pages) raise(TQE_ERR_STATE, "attention was given no pages of the cache");
        const int64_t n = x.rows();
        const int dtype = x.lazy ? BF16 : x.x.dtype;
        const StepContext::Table& table = c.tables.at((size_t)entry.group);
        Tensor q = c.alloc(dtype, {n, n_heads_, head_dim_});
        const int n_pages = (int)entry.keys.shape[0];
        Tensor head_scale;
        if (entry.writes != own_kv_ && !own_kv_) raise(TQE_ERR_STATE, "attention: a layer without keys and values of its own was given a cache of its own");
        if (projected_) {
            if (x.lazy) raise(TQE_ERR_STATE, "attention: this configuration takes no folded norm");
            if (gated_) head_scale = c.alloc(F32, {n, n_heads_});
            projected_q(c, x.x, entry, table, q, head_scale);
        } else if (extras_) {
            if (x.lazy && !turned_first_) raise(TQE_ERR_STATE, "attention: this configuration takes no folded norm");
            if (turned_first_) turned_qkv(c, x, entry, table, q);
            else normed_qkv(c, x.x, entry, table, q);
        } else if (x.lazy || (c.fuse_small && entry.writes && fused_qkv_ok(c))) {
            if (x.lazy && !entry.writes) raise(TQE_ERR_STATE, "a run that reads another run's cache cannot take a folded norm");
            const Position::Tables tb = position_->tables();
            const Tensor& xin = x.lazy ? x.norm.xw : x.x;
            int packed = 0;
            const void* wp = w_qkv_.packed ? (packed = 1, w_qkv_.packed->t.data) : w_qkv_.rows->t.data;
            K::fused_qkv(xin.data, x.lazy ? (const float*)x.norm.ss.data : nullptr, x.lazy ? x.norm.n_ss : 0, x.lazy ? x.norm.eps : 0.f, wp, packed,
                         b_qkv_ ? b_qkv_->t.data : nullptr, (const float*)tb.cos.data, (const float*)tb.sin.data, (int)tb.cos.shape[0], c.dev.tok_pos,
                         table.dev, table.width, entry.keys.data, entry.values.data, n_pages, q.data, (int)n, n_heads_, n_kv_heads_, head_dim_,
                         (int)hidden_, c.stream);
        } else {
            qkv(c, x.x, entry, table, q);
        }
        const int64_t qd = (int64_t)n_heads_ * value_dim_;
        if (last_rows) {
            if (c.n_last == 0) return Tensor(nullptr, dtype, {0, hidden_});
            Tensor ql = c.alloc(dtype, {c.n_last, n_heads_, head_dim_});
            k_gather_rows(c, q, c.dev.last_rows, c.n_last, ql);
            Tensor scale_l;
            if (head_scale.defined()) {
                scale_l = c.alloc(F32, {c.n_last, n_heads_});
                k_gather_rows(c, head_scale, c.dev.last_rows, c.n_last, scale_l);
            }
            Tensor y = c.alloc(dtype, {c.n_last, qd});
            attend_rows(c, ql, entry, table, scale_l, y);
            return linear(c, y, w_o_, b_o_ ? &b_o_->t : nullptr, dtype).t;
        }
        Tensor y = c.alloc(dtype, {n, qd});
        attend(c, q, entry, table, head_scale, y);
        if (stream) {
            add_product(c, *stream, y, w_o_);
            return Tensor();
        }
        return linear(c, y, w_o_, b_o_ ? &b_o_->t : nullptr, dtype).t;
    }

private:
    // product, then biases, the heads' norm, rotation, value mixing and cache write in one kernel
    void normed_qkv(StepContext& c, const Tensor& x, const CacheEntry& entry, const StepContext::Table& table, Tensor& q) {
        const int64_t n = x.shape[0];
        Product p = linear(c, x, w_qkv_, nullptr, x.dtype);
        const Position::Tables tb = position_->tables();
        const bool turn = tb.style != STYLE_NONE;
        const int64_t vd = (int64_t)n_kv_heads_ * value_dim_;
        const void* mix_with = nullptr;
        void* mix_keep = nullptr;
        if (value_mix_ == MIX_SOURCE && entry.writes) {
            Tensor kept(c.ws->alloc_for_step((size_t)(n * vd) * dtype_size(x.dtype)), x.dtype, {n, vd});
            c.carried[mix_key_] = kept;
            mix_keep = kept.data;
        } else if (value_mix_ == MIX_MIXED && entry.writes) {
            auto it = c.carried.find(mix_key_);
            if (it == c.carried.end()) raise(TQE_ERR_STATE, "attention: values are to be mixed with those of an earlier layer, and none has left any in this step");
            if (it->second.dtype != x.dtype || it->second.shape[0] != n || it->second.shape[1] != vd)
                raise(TQE_ERR_STATE, "attention: the values an earlier layer left are %s, wanted [%lld, %lld]", it->second.describe().c_str(), (long long)n, (long long)vd);
            mix_with = it->second.data;
        }
        const int w_dtype = q_norm_ ? q_norm_->t.dtype : mix_ ? mix_->t.dtype : b_qkv_ ? b_qkv_->t.dtype : x.dtype;
        if ((q_norm_ && k_norm_->t.dtype != w_dtype) || (mix_ && mix_->t.dtype != w_dtype) || (b_qkv_ && b_qkv_->t.dtype != w_dtype))
            raise(TQE_ERR_STATE, "attention: the heads' norm weights, the biases and the mixing scalar are of different types");
        const bool write = entry.writes;
        K::normed_rope_store(p.t.data, p.t.dtype, b_qkv_ ? b_qkv_->t.data : nullptr, q_norm_ ? q_norm_->t.data : nullptr, k_norm_ ? k_norm_->t.data : nullptr, w_dtype, eps_,
                             turn ? (const float*)tb.cos.data : nullptr, turn ? (const float*)tb.sin.data : nullptr, turn ? tb.rot_dim : 0,
                             turn ? tb.style : 0, turn ? (int)tb.cos.shape[0] : 0, mix_ ? mix_->t.data : nullptr, mix_with, mix_keep, c.dev.tok_seq, c.dev.tok_pos,
                             write ? table.dev : nullptr, write ? table.width : 0, write ? entry.keys.data : nullptr, write ? entry.values.data : nullptr,
                             q.data, (int)n, n_heads_, n_kv_heads_, head_dim_, value_dim_, write ? 1 : 0, values_are_keys_ ? 1 : 0, c.stream);
    }

    // product (the gate's rows behind the others), then biases, the norm over the projection, rotation, the gate's sigmoid and the cache write
    // in one kernel
    void projected_q(StepContext& c, const Tensor& x, const CacheEntry& entry, const StepContext::Table& table, Tensor& q, Tensor& head_scale) {
        const Tensor p = linear(c, x, w_qkv_, nullptr, x.dtype).t;
        const Position::Tables tb = position_->tables();
        const bool turn = tb.style != STYLE_NONE, write = entry.writes;
        const long long gate_at = (long long)n_heads_ * head_dim_ + (own_kv_ ? (long long)n_kv_heads_ * (head_dim_ + value_dim_) : 0);
        auto floats = [](const OwnedPtr& o) { return o ? (const float*)o->t.data : nullptr; };
        K::projection_store(p.data, p.dtype, row_, floats(bias_f_), floats(q_norm_f_), floats(k_norm_f_), eps_, turn ? (const float*)tb.cos.data : nullptr,
                            turn ? (const float*)tb.sin.data : nullptr, turn ? tb.rot_dim : 0, turn ? tb.style : 0, turn ? (int)tb.cos.shape[0] : 0, c.dev.tok_seq,
                            c.dev.tok_pos, write ? table.dev : nullptr, write ? table.width : 0, write ? entry.keys.data : nullptr,
                            write ? entry.values.data : nullptr, q.data, (float*)head_scale.data, gate_at, (int)x.shape[0], n_heads_, n_kv_heads_, head_dim_,
                            value_dim_, write ? 1 : 0, c.stream);
    }

    // product, then biases, rotation (halves or pairs), the heads' norm without a weight after it, and the cache write in one kernel
    void turned_qkv(StepContext& c, const Activation& x, const CacheEntry& entry, const StepContext::Table& table, Tensor& q) {
        const int64_t n = x.rows();
        Product p;
        if (x.lazy) p.t = linear_of_norm(c, x.norm, w_qkv_, BF16);
        else p = linear(c, x.x, w_qkv_, nullptr, x.x.dtype);
        const Position::Tables tb = position_->tables();
        const bool turn = tb.style != STYLE_NONE;
        const bool write = entry.writes;
        K::rope_norm_store(p.t.data, p.t.dtype, b_qkv_ ? b_qkv_->t.data : nullptr, b_qkv_ ? b_qkv_->t.dtype : 0, turn ? (const float*)tb.cos.data : nullptr,
                           turn ? (const float*)tb.sin.data : nullptr, turn ? tb.rot_dim : 0, turn ? tb.style : 0, turn ? (int)tb.cos.shape[0] : 0,
                           qk_norm_ ? 1 : 0, eps_, c.dev.tok_seq, c.dev.tok_pos, write ? table.dev : nullptr, write ? table.width : 0,
                           write ? entry.keys.data : nullptr, write ? entry.values.data : nullptr, q.data, (int)n, n_heads_, n_kv_heads_, head_dim_, value_dim_,
                           write ? 1 : 0, c.stream);
    }

    // Attention of rows (sequence tok_seq[r], position tok_pos[r]) with the cap, the kept first positions, the sink and the heads' gates.  bfloat16 on the
    // matrix cores where the sizes allow: steps of one token a sequence and a few chosen rows with a row's pages dealt out to
    // partitions, other steps in tiles of consecutive queries; else the plain kernel, one wave per (row, head).
    void attend_masked(StepContext& c, const Tensor& q, const CacheEntry& entry, const StepContext::Table& table, const int32_t* tok_seq,
                       const int32_t* tok_pos, const Tensor& head_scale, Tensor& out, bool last_rows) {
        const int n = (int)q.shape[0], n_pages = (int)entry.keys.shape[0];
        const void* sink = sink_ ? sink_->t.data : nullptr;
        const int sink_dtype = sink_ ? sink_->t.dtype : 0;
        const float* hs = (const float*)head_scale.data;
        if (q.dtype == BF16 && K::attention_masked_mfma_supported.raw(head_dim_, value_dim_)) {
            const bool rows = last_rows ? n <= DECODE_KERNEL_ROWS : c.all_decode;
            if (rows && policy().decode_mfma) {
                const int32_t* row_table = table.dev;
                if (last_rows) {
                    Tensor gathered = c.alloc(I32, {n, table.width});
                    Tensor whole((void*)table.dev, I32, {c.n_seqs, table.width});
                    k_gather_rows(c, whole, c.dev.last_seq, n, gathered);
                    row_table = (const int32_t*)gathered.data;
                }
                // (no more pages than a chunk can touch are ever visited)
                const int n_parts = partitions(n, chunk_ > 0 ? std::min(table.width, (chunk_ + TQE_PAGE - 2) / TQE_PAGE + 1) : table.width);
                Tensor part_out, part_ml;
                if (n_parts > 1) {
                    part_out = c.alloc(F32, {n, n_heads_, n_parts, value_dim_});
                    part_ml = c.alloc(F32, {n, n_heads_, n_parts, 2});
                }
                K::attention_masked_mfma(q.data, entry.keys.data, entry.values.data, tok_pos, row_table, table.width, n_pages, window_, chunk_, keep_first_, scale_,
                                         cap_, sink, sink_dtype, hs, nullptr, nullptr, nullptr, 0, 0, n, n_parts, part_out.data, part_ml.data, out.data, n_heads_,
                                         n_kv_heads_, head_dim_, value_dim_, c.stream);
                return;
            }
            // keys and values of one size, every earlier position visible (or a plain window): the prompt kernel of the plain
            // attention takes the cap, the sink and the heads' gates as options
            if (!rows && policy().prefill_mfma && value_dim_ == head_dim_ && keep_first_ == 0 && scale_ > 0.f &&
                K::attention_prefill_supported.raw(head_dim_)) {
                const int tile = tile_for(c);
                const Tiles t = last_rows ? c.last_tiles(tile) : c.query_tiles(tile);
                K::attention_prefill_capped(q.data, entry.keys.data, entry.values.data, tok_pos, table.dev, table.width, c.n_seqs, n_pages, t.seq, t.tok0,
                                            t.count, t.n, tile, c.dev.seq_start, c.dev.seq_new, window_, chunk_, scale_, cap_, sink, sink_dtype, hs, out.data, n,
                                            n_heads_, n_kv_heads_, head_dim_, c.stream);
                return;
            }
            if (!rows && policy().prefill_mfma) {
                const int tile = K::attention_masked_mfma_tile.raw(n, n_heads_, n_kv_heads_, head_dim_, value_dim_);
                const Tiles t = last_rows ? c.last_tiles(tile) : c.query_tiles(tile);
                K::attention_masked_mfma(q.data, entry.keys.data, entry.values.data, tok_pos, table.dev, table.width, n_pages, window_, chunk_, keep_first_, scale_,
                                         cap_, sink, sink_dtype, hs, t.seq, t.tok0, t.count, t.n, tile, 0, 1, nullptr, nullptr, out.data, n_heads_, n_kv_heads_,
                                         head_dim_, value_dim_, c.stream);
                return;
            }
        }
        K::attention_masked(q.data, entry.keys.data, entry.values.data, q.dtype, tok_seq, tok_pos, table.dev, table.width, c.n_seqs,
                            (int)entry.keys.shape[0], window_, chunk_, keep_first_, scale_, cap_, sink_ ? sink_->t.data : nullptr, sink_ ? sink_->t.dtype : 0,
                            hs, out.data, (int)q.shape[0], n_heads_, n_kv_heads_, head_dim_, value_dim_, c.stream);
    }

    // queries per tile of the prompt kernel for this step
    int tile_for(StepContext& c) const {
        if (prompt_tile_) return prompt_tile_;
        const std::string key = format("prompt_tile:%d:%d:%d", n_heads_, n_kv_heads_, head_dim_);
        auto it = c.memo.find(key);
        if (it == c.memo.end()) it = c.memo.emplace(key, K::attention_prefill_tile.raw(c.n_tokens, n_heads_, n_kv_heads_, head_dim_)).first;
        return it->second;
    }

    // product, then bias, position encoding and cache write in their own kernel
    void qkv(StepContext& c, const Tensor& x, const CacheEntry& entry, const StepContext::Table& table, Tensor& q) {
        const bool own = position_->has_apply();
        const int64_t n = x.shape[0];
        const int total = (n_heads_ + 2 * n_kv_heads_) * head_dim_;
        const int n_pages = (int)entry.keys.shape[0];
        Position::Tables tb;
        bool sums_ok = false;
        if (!own) {
            tb = position_->tables();
            sums_ok = x.dtype == BF16 && K::rope_store_takes_sums.raw(BF16, b_qkv_ ? 1 : 0, b_qkv_ ? b_qkv_->t.dtype : 0, tb.rot_dim, tb.style, head_dim_) != 0;
        }
        Product p = linear(c, x, w_qkv_, nullptr, x.dtype, sums_ok);        // may come as its sums over pieces of K
        const void* bias = nullptr;
        int bias_dt = 0;
        if (own) {
            // a position encoding of its own: bias first, then it changes q and k in place
            if (b_qkv_) K::add_bias(p.t.data, p.t.dtype, b_qkv_->t.data, b_qkv_->t.dtype, (int)n, total, c.stream);
            Tensor qv(p.t.data, p.t.dtype, {n, n_heads_, head_dim_});
            Tensor kv((char*)p.t.data + (size_t)n_heads_ * head_dim_ * dtype_size(p.t.dtype), p.t.dtype, {n, n_kv_heads_, head_dim_});
            position_->apply(c, qv, kv, total);
        } else if (b_qkv_) {
            bias = b_qkv_->t.data;
            bias_dt = b_qkv_->t.dtype;
        }
        const float* cos = tb.style != STYLE_NONE ? (const float*)tb.cos.data : nullptr;
        const float* sin = tb.style != STYLE_NONE ? (const float*)tb.sin.data : nullptr;
        const int max_pos = tb.style != STYLE_NONE ? (int)tb.cos.shape[0] : 0;
        const bool write = entry.writes;
        if (p.is_sums)
            K::rope_store_sums((const float*)p.sums.sums.data, (int)p.sums.sums.shape[0], bias, bias_dt, cos, sin, tb.rot_dim, tb.style, max_pos,
                               c.dev.tok_seq, c.dev.tok_pos, write ? table.dev : nullptr, write ? table.width : 0, write ? c.n_seqs : 0,
                               write ? entry.keys.data : nullptr, write ? entry.values.data : nullptr, write ? n_pages : 0, q.data, (int)n, n_heads_,
                               n_kv_heads_, head_dim_, write ? 1 : 0, c.stream);
        else
            K::rope_store(p.t.data, p.t.dtype, bias, bias_dt, cos, sin, tb.rot_dim, tb.style, max_pos, c.dev.tok_seq, c.dev.tok_pos,
                          write ? table.dev : nullptr, write ? table.width : 0, write ? c.n_seqs : 0, write ? entry.keys.data : nullptr,
                          write ? entry.values.data : nullptr, write ? n_pages : 0, q.data, (int)n, n_heads_, n_kv_heads_, head_dim_, write ? 1 : 0,
                          c.stream);
    }

    // how many partitions a row's pages are dealt out to in the kernels for steps of one token a sequence
    int partitions(int n, int width) const {
        const int q_blocks = (n_heads_ / n_kv_heads_ + 15) / 16;
        const int groups = std::max(1, n * n_kv_heads_ * q_blocks);
        int n_parts = std::max(1, std::min((width + 3) / 4, 256 / groups));
        if (width > 1 && (long long)groups * width <= 640) n_parts = width;
        return n_parts;
    }

    void decode_kernel(StepContext& c, const Tensor& q, const CacheEntry& entry, const int32_t* tok_pos, const int32_t* table, int width,
                       Tensor& out) {
        const int n = (int)q.shape[0];
        const int q_blocks = (n_heads_ / n_kv_heads_ + 15) / 16;
        const int groups = std::max(1, n * n_kv_heads_ * q_blocks);
        const int target_blocks = 256;
        // partitions take the live pages in turn, four waves each: no more than a quarter of the pages there can be
        // (more partitions than one block per compute unit, so that no wave has a second page to bring in, measured
        // slower: 14.6 against 13.8 us for 8 sequences of 2100 positions at the 7B sizes; 64 sequences in 2 and 4
        // partitions 60.6 and 65.9 against 56.4 us, 128 sequences 118 and 133 against 114).  Nor fewer, larger blocks
        // that need no merge: one block of eight waves per (sequence, kv head) took 37 us for the 8 sequences, since a
        // compute unit alone pulls about 30 GB/s whatever its waves ask for.
        // (no more blocks than compute units: with 288 blocks 32 units get two, and 12 sequences took 19.5 us against
        // 16.1 with 240 blocks, 24 sequences 32.2 against 27.0, 48 sequences 48.9 + merge against 40.8 without)
        int n_parts = std::max(1, std::min((width + 3) / 4, target_blocks / groups));
        // few sequences: a partition per page of the table, which the kernel gives a block of one wave each (faster up to
        // four sequences of 2100 positions at the 7B sizes, slower from eight on)
        if (width > 1 && (long long)groups * width <= 640) n_parts = width;
        Tensor part_out, part_ml;
        if (n_parts > 1) {
            part_out = c.alloc(F32, {n, n_heads_, n_parts, head_dim_});
            part_ml = c.alloc(F32, {n, n_heads_, n_parts, 2});
        }
        K::attention_decode(q.data, entry.keys.data, entry.values.data, tok_pos, table, width, n, (int)entry.keys.shape[0], window_, scale_, n_parts,
                            part_out.data, part_ml.data, out.data, n_heads_, n_kv_heads_, head_dim_, c.stream);
    }

    // Softmax attention of q over the cache entry: picks the kernel for the step.  float32, or a
    // head size the MFMA kernels do not take: the plain kernel, one wave per (token, head).
    // bfloat16 and one token per sequence: the partitioned decoding kernel; bfloat16 otherwise: the
    // tiled prompt kernel.
    void attend(StepContext& c, const Tensor& q, const CacheEntry& entry, const StepContext::Table& table, const Tensor& head_scale, Tensor& out) {
        const int n = (int)q.shape[0], n_pages = (int)entry.keys.shape[0];
        if (extras_) return attend_masked(c, q, entry, table, c.dev.tok_seq, c.dev.tok_pos, head_scale, out, false);
        if (q.dtype == BF16 && c.all_decode && policy().decode_mfma && K::attention_decode_supported.raw(head_dim_))
            return decode_kernel(c, q, entry, c.dev.tok_pos, table.dev, table.width, out);
        // (not for steps of one token per sequence: tiles of one query are what the plain kernel does anyway,
        // and such a step may be replayed from a graph, which cannot carry the tiles' upload)
        if (q.dtype == BF16 && !c.all_decode && policy().prefill_mfma && scale_ > 0.f && K::attention_prefill_supported.raw(head_dim_)) {
            const int tile = tile_for(c);
            const Tiles t = c.query_tiles(tile);
            K::attention_prefill(q.data, entry.keys.data, entry.values.data, c.dev.tok_pos, table.dev, table.width, c.n_seqs, n_pages, t.seq, t.tok0,
                                 t.count, t.n, tile, c.dev.seq_start, c.dev.seq_new, window_, scale_, out.data, n, n_heads_, n_kv_heads_, head_dim_,
                                 c.stream);
            return;
        }
        K::attention(q.data, entry.keys.data, entry.values.data, q.dtype, c.dev.tok_seq, c.dev.tok_pos, table.dev, table.width, c.n_seqs, n_pages,
                     window_, scale_, out.data, n, n_heads_, n_kv_heads_, head_dim_, c.stream);
    }

    // The same for the step's last_rows alone (q holds their queries): the cache already holds the
    // keys and values of all the step's tokens.
    void attend_rows(StepContext& c, const Tensor& q, const CacheEntry& entry, const StepContext::Table& table, const Tensor& head_scale, Tensor& out) {
        const int n = (int)q.shape[0], n_pages = (int)entry.keys.shape[0];
        if (extras_) return attend_masked(c, q, entry, table, c.dev.last_seq, c.dev.last_pos, head_scale, out, true);
        if (q.dtype == BF16 && policy().decode_mfma && K::attention_decode_supported.raw(head_dim_) && c.n_last <= DECODE_KERNEL_ROWS) {
            // few rows: the decoding kernel shares a row's keys out over many blocks, where the prompt
            // kernel would walk them in one; a row is a sequence of its own to it
            Tensor rows_table = c.alloc(I32, {n, table.width});
            Tensor whole((void*)table.dev, I32, {c.n_seqs, table.width});
            k_gather_rows(c, whole, c.dev.last_seq, n, rows_table);
            return decode_kernel(c, q, entry, c.dev.last_pos, (const int32_t*)rows_table.data, table.width, out);
        }
        if (q.dtype == BF16 && policy().prefill_mfma && scale_ > 0.f && K::attention_prefill_supported.raw(head_dim_)) {
            const int tile = tile_for(c);
            const Tiles t = c.last_tiles(tile);
            K::attention_prefill(q.data, entry.keys.data, entry.values.data, c.dev.last_pos, table.dev, table.width, c.n_seqs, n_pages, t.seq, t.tok0,
                                 t.count, t.n, tile, c.dev.seq_start, c.dev.seq_new, window_, scale_, out.data, n, n_heads_, n_kv_heads_, head_dim_,
                                 c.stream);
            return;
        }
        K::attention(q.data, entry.keys.data, entry.values.data, q.dtype, c.dev.last_seq, c.dev.last_pos, table.dev, table.width, c.n_seqs, n_pages,
                     window_, scale_, out.data, n, n_heads_, n_kv_heads_, head_dim_, c.stream);
    }

    int act_dtype_;
    int64_t hidden_;
    int n_heads_, n_kv_heads_, head_dim_, window_, prompt_tile_;
    bool qkv_bias_, out_bias_;
    float scale_;
    enum { MIX_NONE = 0, MIX_SOURCE = 1, MIX_MIXED = 2 };
    int value_dim_, chunk_ = 0, keep_first_, value_mix_ = MIX_NONE;
    bool qk_norm_ = false, has_sink_ = false, extras_ = false, cache_keeps_all_ = false, values_are_keys_ = false;
    bool qk_norm_weight_ = true, norm_after_rotation_ = false, turned_first_ = false;
    bool projected_ = false, fixed_sink_ = false, gated_ = false, own_kv_ = true;
    int cache_window_ = 0;
    int64_t row_ = 0;
    float eps_ = 0.f, cap_ = 0.f, sink_score_ = 0.f;
    std::string n_gate_;
    OwnedPtr bias_f_, q_norm_f_, k_norm_f_;
    std::string mix_key_, n_q_, n_k_, n_v_, n_o_, n_q_norm_, n_k_norm_, n_sink_, n_mix_, n_qb_, n_kb_, n_vb_;
    std::shared_ptr<Position> position_;
    Weight w_qkv_, w_o_;
    OwnedPtr b_qkv_, b_o_, q_norm_, k_norm_, sink_, mix_;
};

// ---- gated feed-forward ----------------------------------------------------------------------------
// down(gate(gate_proj(x), up_proj(x))), no biases.  With the SiLU gate this is "SwiGLU" as the reference's Mlp
// (src/models/turbo_generic.rs:98-111): down(silu(gate(x)) * up(x)); kind "gated_silu" is that.  Kind "gated"
// names its gate (params gate: silu, relu, clamped with limit and alpha, gelu_tanh; see Gate in linear.h).  Gate
// and up are one product with the weights stacked.  params: hidden, inter; optional names {gate, up, down}: the
// three tensors' names inside the part's prefix.
class GatedSiLU : public FeedForward {
public:
    GatedSiLU(const PartSpec& spec, BuildEnv&, bool any_gate) {
        KeyReader r(spec.params, any_gate ? "gated" : "gated_silu", TQE_ERR_ARGUMENT);
        hidden_ = r.integer("hidden", 1);
        inter_ = r.integer("inter", 1);
        if (any_gate) gate_ = Gate::from_params(r, "gated");
        const Json& names = spec.params["names"];
        auto name = [&](const char* role, const char* fallback) { return names[role].is_string() ? names[role].as_string() : std::string(fallback); };
        n_gate_ = name("gate", "gate_proj.weight");
        n_up_ = name("up", "up_proj.weight");
        n_down_ = name("down", "down_proj.weight");
        graph_safe = true;
    }
    TensorSpecs tensors() const override {
        auto w = [](int64_t a, int64_t b) { TensorSpec t; t.shape = {a, b}; return t; };
        return {{n_gate_, w(inter_, hidden_)}, {n_up_, w(inter_, hidden_)}, {n_down_, w(hidden_, inter_)}};
    }
    void load(Loaded& t, hipStream_t stream) override {
        OwnedPtr gu = stack_rows({take(t, n_gate_.c_str()), take(t, n_up_.c_str())}, stream);
        w_gate_up_ = make_weight(gu, 2, false, stream);
        w_down_ = make_weight(take(t, n_down_.c_str()), 1, false, stream);
    }
    OwnedPtr held(const std::string& name) const override {
        if (name == "gate_up.weight") return w_gate_up_.rows;
        if (name == "gate_up.weight.packed") return w_gate_up_.packed;
        if (name == "down_proj.weight") return w_down_.rows;
        if (name == "down_proj.weight.packed") return w_down_.packed;
        return nullptr;
    }
    const char* trace_name() const override { return "attn-mlp"; }         // the reference's span, src/models/turbo_generic.rs:1922
    void product_shapes(std::vector<std::pair<int64_t, int64_t>>& out) const override {
        out.push_back({2 * inter_, hidden_});
        out.push_back({hidden_, inter_});
    }

    bool folds_norm(const StepContext& c) const override { return fusable(c.n_tokens, w_gate_up_); }
    bool adds_to_stream(const StepContext& c) const override {
        return (fusable(c.n_tokens, w_down_, true) && fusable(c.n_tokens, w_gate_up_)) || leaves_sums(c.n_tokens, w_down_);
    }

    Tensor forward(StepContext& c, const Activation& x, Stream* stream) override {
        if (stream && !x.lazy && x.x.shape[0] > skinny_max_rows()) {
            add_product(c, *stream, gated_linear(c, x.x, w_gate_up_, gate_), w_down_);
            return Tensor();
        }
        if (x.lazy || stream) {
            const Tensor& xin = x.lazy ? x.norm.xw : x.x;
            Tensor act = c.alloc(BF16, {xin.shape[0], inter_});
            int packed = 0;
            const void* wp = w_gate_up_.packed ? (packed = 1, w_gate_up_.packed->t.data) : w_gate_up_.rows->t.data;
            K::fused_gated_act(xin.data, x.lazy ? (const float*)x.norm.ss.data : nullptr, x.lazy ? x.norm.n_ss : 0, x.lazy ? x.norm.eps : 0.f, wp,
                               packed, act.data, (int)xin.shape[0], (int)(2 * inter_), (int)hidden_, gate_.kind, gate_.limit, gate_.alpha, c.stream);
            if (!stream) return linear(c, act, w_down_, nullptr, BF16).t;
            add_product(c, *stream, act, w_down_);
            return Tensor();
        }
        return linear(c, gated_linear(c, x.x, w_gate_up_, gate_), w_down_, nullptr, x.x.dtype).t;
    }

private:
    int64_t hidden_, inter_;
    Gate gate_;
    std::string n_gate_, n_up_, n_down_;
    Weight w_gate_up_, w_down_;
};

// ---- the pre-norm block ----------------------------------------------------------------------------
// The reference's decoder layer (src/models/turbo_generic.rs:1959-1981): x = x + mixer(norm(x));
// x = x + ff(norm(x)), with optional norms on the mixer's and the feed-forward's outputs
// (:1965-1968, :1976-1979).
//
// The residual stream is float32.  A part's output is left pending on the stream and added inside
// the next norm's kernel (for mid-sized steps a part's last product may even leave its sums over
// pieces of K pending: the norm's kernel adds those up too).  In small decoding steps the
// framework's parts go further: a product that consumes a norm computes it itself (LazyNorm) and a
// part's last product adds its result to the stream in its epilogue, so that the norm kernels
// disappear; parts that do not offer this are simply given tensors.  An output norm (post_mixer_norm, post_ff_norm) whose kind the
// next norm knows is left to that norm's kernel too: output norm, sum and next norm are one pass.
//
// params: mixer, feed_forward, mixer_norm, ff_norm (part specs); optional post_mixer_norm,
// post_ff_norm; names: part -> tensor-name prefix inside the layer (e.g. {"mixer": "self_attn."}).
class PreNormBlock : public Block {
public:
    PreNormBlock(const PartSpec& spec, BuildEnv& env) {
        const Json& names = spec.params["names"];
        auto one = [&](const char* role, const char* category, bool optional) -> std::shared_ptr<Part> {
            const Json& p = spec.params[role];
            if (p.is_null()) {
                if (optional) return nullptr;
                raise(TQE_ERR_ARGUMENT, "pre_norm block: no '%s' given", role);
            }
            std::shared_ptr<Part> part = build_part(category, PartSpec::from_json(p, role), env);
            if (!names[role].is_string()) raise(TQE_ERR_ARGUMENT, "pre_norm block: no tensor-name prefix for '%s'", role);
            roles_.push_back({role, names[role].as_string(), part});
            return part;
        };
        mixer_ = std::dynamic_pointer_cast<Mixer>(one("mixer", "mixer", false));
        // a layer may have no feed-forward (feed_forward: null): then it has no norm in front of one either
        const bool has_ff = !spec.params["feed_forward"].is_null();
        feed_forward_ = std::dynamic_pointer_cast<FeedForward>(one("feed_forward", "feed_forward", true));
        mixer_norm_ = std::dynamic_pointer_cast<Norm>(one("mixer_norm", "norm", false));
        ff_norm_ = has_ff ? std::dynamic_pointer_cast<Norm>(one("ff_norm", "norm", false)) : nullptr;
        post_mixer_norm_ = std::dynamic_pointer_cast<Norm>(one("post_mixer_norm", "norm", true));
        post_ff_norm_ = has_ff ? std::dynamic_pointer_cast<Norm>(one("post_ff_norm", "norm", true)) : nullptr;
        if (!mixer_ || (has_ff && (!feed_forward_ || !ff_norm_)) || !mixer_norm_) raise(TQE_ERR_ARGUMENT, "pre_norm block: a part is of the wrong category");
        graph_safe = true;
        for (const Role& r : roles_) graph_safe = graph_safe && r.part->graph_safe;
    }
    TensorSpecs tensors() const override {
        TensorSpecs out;
        for (const Role& r : roles_)
            for (const auto& t : r.part->tensors()) out.push_back({r.prefix + t.first, t.second});
        return out;
    }
    void load(Loaded& tensors, hipStream_t stream) override {
        for (const Role& r : roles_) {
            Loaded own;
            for (const auto& t : r.part->tensors()) own[t.first] = take(tensors, (r.prefix + t.first).c_str());
            r.part->load(own, stream);
        }
    }
    OwnedPtr held(const std::string& name) const override {
        for (const Role& r : roles_)
            if (name.compare(0, r.prefix.size(), r.prefix) == 0)
                if (OwnedPtr p = r.part->held(name.substr(r.prefix.size()))) return p;
        return nullptr;
    }
    Json describe() const override {
        Json j = Part::describe();
        Json parts = Json::object();
        for (const Role& r : roles_) parts.set(r.role, r.part->describe());
        j.set("parts", parts);
        return j;
    }
    void product_shapes(std::vector<std::pair<int64_t, int64_t>>& out) const override {
        for (const Role& r : roles_) r.part->product_shapes(out);
    }
    CacheNeed cache_need() const override { return mixer_->cache_need(); }
    Norm* first_norm() override { return mixer_norm_.get(); }
    Mixer* mixer() override { return mixer_.get(); }

    Stream* forward(StepContext& c, Stream* stream, const CacheEntry& entry, Norm* next_norm, bool last) override {
        if (last && c.prune_last && policy().prune_last && mixer_->takes_rows) return forward_last_rows(c, stream, entry, next_norm);
        Activation x = normed(c, *mixer_norm_, *stream, mixer_->folds_norm(c));
        {
            Span span(mixer_->trace_name());
            Norm* reader = feed_forward_ ? ff_norm_.get() : next_norm;
            const bool adds = may_add(c, post_mixer_norm_.get(), reader) && mixer_->adds_to_stream(c);
            if (adds) stream->next_norm = reader;
            settle(c, *stream, mixer_->forward(c, x, entry, adds ? stream : nullptr, false), post_mixer_norm_.get(), reader);
        }
        if (!feed_forward_) return stream;
        x = normed(c, *ff_norm_, *stream, feed_forward_->folds_norm(c));
        {
            Span span(feed_forward_->trace_name());
            const bool adds = may_add(c, post_ff_norm_.get(), next_norm) && feed_forward_->adds_to_stream(c);
            if (adds) stream->next_norm = next_norm;
            settle(c, *stream, feed_forward_->forward(c, x, adds ? stream : nullptr), post_ff_norm_.get(), next_norm);
        }
        return stream;
    }

private:
    struct Role { std::string role, prefix; std::shared_ptr<Part> part; };

    // the part's input: the norm of the stream, computed now, or left to the part
    Activation normed(StepContext& c, Norm& norm, Stream& stream, bool part_folds) {
        Activation a;
        if (c.fuse_small && part_folds && norm.lazy(stream, a.norm)) {
            a.lazy = true;
            return a;
        }
        Span span(norm.trace_name());
        a.x = c.alloc(c.act_dtype, {stream.h.shape[0], stream.h.shape[1]});
        norm.add_norm(c, stream.h, stream.pending, a.x);
        stream.pending = Pending();
        stream.invalidate();
        return a;
    }
    // Whether a part may be given the stream.  With an output norm it must not be added yet: only in steps whose products are left pending
    // (as sums over pieces of K), for a next norm that applies the output norm first.
    static bool may_add(const StepContext& c, const Norm* post_norm, const Norm* next_norm) {
        if (!post_norm) return c.fuse_small || c.fuse_mid;
        return c.fuse_mid && next_norm && next_norm->takes_normed_update(post_norm) && next_norm->takes_partial_sums();
    }
    // a part's output that it did not add to the stream itself is left pending for the next norm's kernel
    // (an output norm that goes with the next norm's kernel: what a part left pending on the stream is that norm's to read)
    void settle(StepContext& c, Stream& stream, Tensor out, Norm* post_norm, const Norm* next_norm) {
        if (!out.defined()) {
            if (post_norm) stream.pending.norm = post_norm;
            return;
        }
        const bool together = post_norm && next_norm && next_norm->takes_normed_update(post_norm);
        if (post_norm && !together) {
            Tensor y = c.alloc(out.dtype, {out.shape[0], out.shape[1]});
            post_norm->forward(c, out, y);
            out = y;
        }
        stream.pending = Pending::of(out);
        if (together) stream.pending.norm = post_norm;
        stream.invalidate();
    }

    Stream* forward_last_rows(StepContext& c, Stream* stream, const CacheEntry& entry, const Norm* next_norm) {
        Activation x;
        {
            Span span(mixer_norm_->trace_name());
            x.x = c.alloc(c.act_dtype, {stream->h.shape[0], stream->h.shape[1]});
            mixer_norm_->add_norm(c, stream->h, stream->pending, x.x);
        }
        Tensor y;
        {
            Span span(mixer_->trace_name());
            y = mixer_->forward(c, x, entry, nullptr, true);        // keys and values of all tokens, output of the rows
        }
        c.sub_stream.reset(new Stream());
        Stream* sub = c.sub_stream.get();
        sub->of_last_rows = true;
        sub->h = c.alloc(F32, {c.n_last, stream->h.shape[1]});
        if (c.n_last == 0) return sub;
        k_gather_rows(c, stream->h, c.dev.last_rows, c.n_last, sub->h);
        settle(c, *sub, y, post_mixer_norm_.get(), feed_forward_ ? ff_norm_.get() : next_norm);
        if (!feed_forward_) return sub;
        {
            Span span(ff_norm_->trace_name());
            x.x = c.alloc(c.act_dtype, {c.n_last, stream->h.shape[1]});
            ff_norm_->add_norm(c, sub->h, sub->pending, x.x);
            sub->pending = Pending();
        }
        Tensor out;
        {
            Span span(feed_forward_->trace_name());
            out = feed_forward_->forward(c, x, nullptr);
        }
        settle(c, *sub, out, post_ff_norm_.get(), next_norm);
        return sub;
    }

    std::vector<Role> roles_;
    std::shared_ptr<Mixer> mixer_;
    std::shared_ptr<FeedForward> feed_forward_;
    std::shared_ptr<Norm> mixer_norm_, ff_norm_, post_mixer_norm_, post_ff_norm_;
};

void register_builtin_parts() {
    static std::once_flag once;
    std::call_once(once, [] {
        register_kind("norm", "rms_norm", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<RMSNorm>(s, e); });
        register_kind("position", "rotary", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<Rotary>(s, e); });
        register_kind("position", "none", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<NoPosition>(s, e); });
        register_kind("mixer", "attention", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<Attention>(s, e); });
        register_kind("feed_forward", "gated_silu", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<GatedSiLU>(s, e, false); });
        register_kind("feed_forward", "gated", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<GatedSiLU>(s, e, true); });
        register_latent_parts();
        register_moe_parts();
        register_stream_parts();
        register_recurrent_parts();
        register_streams_parts();
        register_linear_attention_parts();
        register_pooled_parts();
        register_mlstm_parts();
        register_time_mixing_parts();
        register_joint_parts();
        register_kind("block", "pre_norm", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<PreNormBlock>(s, e); });
    });
}

}  // namespace tq
