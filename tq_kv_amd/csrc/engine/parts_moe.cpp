// A feed-forward of routed experts.
//
// Each token goes through `top` of `n_experts` small gated feed-forwards.  The router's logits
// z = W_r x are computed in float32, s = softmax(z) runs over all experts, the `top` largest are
// chosen, and their outputs are added up with the weights s * router_scale (not renormalised).  An
// expert is down(gate(gate_proj x, up_proj x)) with the gate its params name (Gate in linear.h); it
// has no biases.  A shared expert (any feed-forward part, optional) runs for every token and is
// added.
//
// The step's (token, expert) pairs are grouped by expert on the device (moe.hip): the products run
// over tiles of rows that belong to one expert, from lists that stay on the device, so the
// launches are the same whatever the router chose and a step can be captured as a graph.
//
// Variants, all parameters: gated false makes an expert down(f(up_proj x)), f the gate's function of one product
// (relu2: max(z, 0)^2), without a gate product and its tensor; normalize "chosen" makes the weights the softmax over
// the chosen logits alone (times router_scale); shared_gate names a tensor [1, hidden] whose product with x, through
// a sigmoid, multiplies the shared expert's output token by token; score "sigmoid" makes an expert's score sigmoid(z) on its own
// instead of the softmax over all; weight_on "input" multiplies an expert's input by the weight (the output is then the plain sum of
// E(w x) over the chosen experts, which is not w E(x) since an expert is not linear).
//
// Choosing by more than the score: correction names a tensor [experts + identity] that is added to the scores for the choice alone;
// n_groups and keep_groups cut the experts into equal groups of neighbours, and only experts of the keep_groups best groups (by the largest
// choice score in them) can be chosen; identity: so many experts more, the router's last, that have no tensors and give back their
// input.  With any of them the weights are the chosen experts' softmax scores over their sum plus weight_floor (normalize "chosen").
//
// params: hidden, inter, n_experts, top, router_scale, gate / limit / alpha, gated, normalize, score, weight_on, identity, correction (a tensor's
// name, or null), n_groups, keep_groups, weight_floor, shared (a feed-forward
// part spec, or null), shared_gate (a tensor's name, or null); optional names {router, expert (with %d for the expert's number), gate, up,
// down, shared}.  Tensors: router [experts + identity, hidden]; per expert gate, up [inter, hidden], down
// [hidden, inter]; the shared expert's own under its prefix.
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

class RoutedExperts : public FeedForward {
public:
    RoutedExperts(const PartSpec& spec, BuildEnv& env) {
        KeyReader r(spec.params, "routed_experts", TQE_ERR_ARGUMENT);
        hidden_ = r.integer("hidden", 1);
        inter_ = r.integer("inter", 1);
        n_experts_ = (int)r.integer("n_experts", 1);
        top_ = (int)r.integer("top", 1);
        router_scale_ = (float)r.number_or("router_scale", 1.0);
        gate_ = Gate::from_params(r, "routed_experts");
        gated_ = r.boolean_or("gated", true);
        const std::string normalize = r.string_or("normalize", "all");
        if (normalize != "all" && normalize != "chosen") raise(TQE_ERR_ARGUMENT, "routed_experts: unknown normalize '%s' (known: all, chosen)", normalize.c_str());
        renormalize_ = normalize == "chosen";
        const std::string score = r.string_or("score", "softmax");
        if (score != "softmax" && score != "sigmoid") raise(TQE_ERR_ARGUMENT, "routed_experts: unknown score '%s' (known: sigmoid, softmax)", score.c_str());
        sigmoid_scores_ = score == "sigmoid";
        const std::string weight_on = r.string_or("weight_on", "output");
        if (weight_on != "output" && weight_on != "input") raise(TQE_ERR_ARGUMENT, "routed_experts: unknown weight_on '%s' (known: input, output)", weight_on.c_str());
        weight_on_input_ = weight_on == "input";
        n_shared_gate_ = r.string_or("shared_gate", "");
        identity_ = (int)r.integer_or("identity", 0, 0);
        n_correction_ = r.string_or("correction", "");
        n_groups_ = (int)r.integer_or("n_groups", 1, 1);
        keep_groups_ = (int)r.integer_or("keep_groups", n_groups_, 1);
        weight_floor_ = (float)r.number_or("weight_floor", 0.0);
        const int outputs = n_experts_ + identity_;
        by_choice_ = identity_ > 0 || !n_correction_.empty() || keep_groups_ < n_groups_ || weight_floor_ != 0.f;
        if (top_ > outputs) raise(TQE_ERR_ARGUMENT, "routed_experts: top %d of %d experts", top_, outputs);
        if (outputs % n_groups_ || keep_groups_ > n_groups_) raise(TQE_ERR_ARGUMENT, "routed_experts: %d of %d groups of %d experts", keep_groups_, n_groups_, outputs);
        if (top_ > keep_groups_ * (outputs / n_groups_))
            raise(TQE_ERR_ARGUMENT, "routed_experts: top %d of the %d experts that %d groups hold", top_, keep_groups_ * (outputs / n_groups_), keep_groups_);
        if (by_choice_ && (!renormalize_ || sigmoid_scores_ || !n_shared_gate_.empty() || router_scale_ != 1.f))
            raise(TQE_ERR_ARGUMENT, "routed_experts: identity, correction, groups and weight_floor go with softmax scores, normalize 'chosen', router_scale 1 and no shared_gate");
        const int most = K::moe_max_experts.raw();
        if (outputs > most) raise(TQE_ERR_CONFIG, "routed_experts: %d experts are more than the kernels take (%d)", outputs, most);
        const Json& names = spec.params["names"];
        auto name = [&](const char* role, const char* fallback) { return names[role].is_string() ? names[role].as_string() : std::string(fallback); };
        n_router_ = name("router", "router");
        n_expert_ = name("expert", "e%d.");
        n_gate_ = name("gate", "gate");
        n_up_ = name("up", "up");
        n_down_ = name("down", "down");
        n_shared_ = name("shared", "shared.");
        if (n_expert_.find("%d") == std::string::npos || n_expert_.find('%') != n_expert_.rfind('%'))
            raise(TQE_ERR_ARGUMENT, "routed_experts: the experts' prefix '%s' must hold one %%d", n_expert_.c_str());
        graph_safe = true;
        if (!spec.params["shared"].is_null()) {
            shared_ = std::dynamic_pointer_cast<FeedForward>(build_part("feed_forward", PartSpec::from_json(spec.params["shared"], "routed_experts: shared"), env));
            if (!shared_) raise(TQE_ERR_ARGUMENT, "routed_experts: the shared expert is no feed-forward");
            graph_safe = shared_->graph_safe;
        }
        if (!n_shared_gate_.empty() && !shared_) raise(TQE_ERR_ARGUMENT, "routed_experts: a gate for a shared expert that is not there");
    }

    std::string expert_prefix(int e) const {
        std::string s = n_expert_;
        s.replace(s.find("%d"), 2, std::to_string(e));
        return s;
    }
    TensorSpecs tensors() const override {
        auto w = [](int64_t a, int64_t b) { TensorSpec t; t.shape = {a, b}; return t; };
        TensorSpecs t = {{n_router_, w(n_experts_ + identity_, hidden_)}};
        if (!n_correction_.empty()) { TensorSpec c; c.shape = {n_experts_ + identity_}; t.push_back({n_correction_, c}); }
        for (int e = 0; e < n_experts_; ++e) {
            const std::string p = expert_prefix(e);
            if (gated_) t.push_back({p + n_gate_, w(inter_, hidden_)});
            t.push_back({p + n_up_, w(inter_, hidden_)});
            t.push_back({p + n_down_, w(hidden_, inter_)});
        }
        if (shared_)
            for (const auto& s : shared_->tensors()) t.push_back({n_shared_ + s.first, s.second});
        if (!n_shared_gate_.empty()) t.push_back({n_shared_gate_, w(1, hidden_)});
        return t;
    }
    void load(Loaded& t, hipStream_t stream) override {
        router_ = take(t, n_router_);
        if (by_choice_) w_router_ = make_weight(router_, 1, true, stream);
        if (!n_correction_.empty()) correction_ = as_floats(stored_correction_ = take(t, n_correction_), stream);
        // all experts' weights in two tensors: [experts, gate rows then up rows, hidden] and [experts, hidden, inter]
        std::vector<OwnedPtr> gu, down;
        for (int e = 0; e < n_experts_; ++e) {
            const std::string p = expert_prefix(e);
            if (gated_) gu.push_back(take(t, p + n_gate_));
            gu.push_back(take(t, p + n_up_));
            down.push_back(take(t, p + n_down_));
        }
        gate_up_ = stack_rows(gu, stream);
        down_ = stack_rows(down, stream);
        if (shared_) {
            Loaded own;
            for (const auto& s : shared_->tensors()) own[s.first] = take(t, n_shared_ + s.first);
            shared_->load(own, stream);
        }
        if (!n_shared_gate_.empty()) shared_gate_ = take(t, n_shared_gate_);
    }
    OwnedPtr held(const std::string& name) const override {
        if (name == n_router_) return router_;
        if (!n_correction_.empty() && name == n_correction_) return stored_correction_;
        if (!n_shared_gate_.empty() && name == n_shared_gate_) return shared_gate_;
        if (name == "experts.gate_up") return gate_up_;
        if (name == "experts.down") return down_;
        if (shared_ && name.compare(0, n_shared_.size(), n_shared_) == 0) return shared_->held(name.substr(n_shared_.size()));
        return nullptr;
    }
    const char* trace_name() const override { return "attn-mlp"; }
    void product_shapes(std::vector<std::pair<int64_t, int64_t>>& out) const override {
        if (shared_) shared_->product_shapes(out);
    }

    Tensor forward(StepContext& c, const Activation& x, Stream*) override { return run(c, x, nullptr, 1.f, nullptr, nullptr); }
    bool takes_beside() const override { return true; }
    Tensor forward_beside(StepContext& c, const Activation& x, const Tensor& beside, float scale, Stream* stream, const Norm* next_norm) override {
        if (beside.dtype != x.x.dtype || beside.shape[0] != x.x.shape[0] || beside.cols() != hidden_)
            raise(TQE_ERR_STATE, "routed_experts: what is to be added is %s for a step of [%lld, %lld]", beside.describe().c_str(), (long long)x.x.shape[0], (long long)hidden_);
        return run(c, x, beside.data, scale, stream, next_norm);
    }

private:
    Tensor run(StepContext& c, const Activation& x, const void* beside, float scale, Stream* stream, const Norm* next_norm) {
        if (x.lazy) raise(TQE_ERR_STATE, "routed_experts takes no folded norm");
        const int64_t n = x.x.shape[0];
        const int dtype = x.x.dtype;
        const int64_t pairs = n * top_;
        // bfloat16 on the matrix cores, in tiles whose size follows the rows an expert gets on average; else the plain kernel
        const bool on_cores = dtype == BF16 && gate_up_->t.dtype == BF16 && down_->t.dtype == BF16 && policy().skinny && hidden_ % 8 == 0 &&
                              inter_ % 8 == 0 && K::grouped_supported.raw((int)hidden_) != 0;
        const int64_t per_expert = pairs / n_experts_;
        const bool big = on_cores && per_expert >= 96 && K::grouped_max_tile.raw((int)inter_, (int)hidden_) >= 128 && K::grouped_max_tile.raw((int)hidden_, (int)inter_) >= 128;
        const int tile_m = !on_cores ? K::moe_tile_rows.raw() : big ? 128 : per_expert >= 48 ? 64 : per_expert >= 24 ? 32 : 16;
        const int max_tiles = K::moe_max_tiles.raw((int)pairs, n_experts_, tile_m);
        Tensor idx = c.alloc(I32, {n, top_}), weight = c.alloc(F32, {n, top_});
        Tensor pair_pos = c.alloc(I32, {pairs}), sorted_tok = c.alloc(I32, {pairs});
        Tensor tiles = c.alloc(I32, {3, max_tiles}), n_tiles = c.alloc(I32, {4});
        int32_t* tile_expert = (int32_t*)tiles.data;
        int32_t* tile_row0 = tile_expert + max_tiles;
        int32_t* tile_rows = tile_row0 + max_tiles;
        // the shared expert's gate rides along with the router where both weights are of one type
        Tensor shared_scale;
        const bool gate_in_route = shared_gate_ && shared_gate_->t.dtype == router_->t.dtype;
        if (shared_gate_) shared_scale = c.alloc(F32, {n});
        const float* correction = correction_ ? (const float*)correction_->t.data : nullptr;
        const int outputs = n_experts_ + identity_;
        if (by_choice_ && dtype == BF16 && router_->t.dtype == BF16 && n > mid_max_rows() && outputs % 8 == 0 && hidden_ % 8 == 0 && policy().library && !null_device()) {
            // steps of many tokens: the logits as a product of bfloat16 operands with float32 sums (which is what the kernel below forms too)
            const Tensor z = linear(c, x.x, w_router_, nullptr, F32).t;
            K::moe_choose_grouped((const float*)z.data, outputs, top_, correction, n_groups_, keep_groups_, weight_floor_, (int32_t*)idx.data, (float*)weight.data, (int)n,
                                  c.stream);
        } else if (by_choice_)
            K::moe_route_grouped(x.x.data, dtype, router_->t.data, router_->t.dtype, outputs, (int)hidden_, top_, correction, n_groups_, keep_groups_, weight_floor_, (int32_t*)idx.data,
                                 (float*)weight.data, (int)n, c.stream);
        else
            K::moe_route(x.x.data, dtype, router_->t.data, router_->t.dtype, n_experts_, (int)hidden_, top_, router_scale_, (renormalize_ ? 1 : 0) | (sigmoid_scores_ ? 2 : 0), (int32_t*)idx.data,
                         (float*)weight.data, gate_in_route ? shared_gate_->t.data : nullptr, gate_in_route ? (float*)shared_scale.data : nullptr, (int)n, c.stream);
        K::moe_group((const int32_t*)idx.data, (int)n, top_, n_experts_, tile_m, (int32_t*)pair_pos.data, (int32_t*)sorted_tok.data, tile_expert, tile_row0,
                     tile_rows, (int32_t*)n_tiles.data, c.stream);
        Tensor shared_out;
        if (shared_) shared_out = shared_->forward(c, x, nullptr);
        if (shared_gate_ && !gate_in_route) {
            K::row_gate(x.x.data, dtype, shared_gate_->t.data, shared_gate_->t.dtype, (float*)shared_scale.data, (int)n, (int)hidden_, c.stream);
        }
        // an expert's first product: gate and up side by side, or up alone with the gate's function of it
        const int first = gated_ ? 1 : 2;
        const long long first_stride = (long long)(gated_ ? 2 : 1) * inter_ * hidden_;
        Tensor act = c.alloc(dtype, {pairs, inter_});
        Tensor y = c.alloc(dtype, {pairs, hidden_});
        // the weight on the experts' inputs: every pair's row is its token's times the pair's weight, and the sum below is a plain one
        const void* first_in = x.x.data;
        const int32_t* first_rows = (const int32_t*)sorted_tok.data;
        const float* sum_weight = (const float*)weight.data;
        if (weight_on_input_) {
            Tensor scaled = c.alloc(dtype, {pairs, hidden_}), unit = c.alloc(F32, {n, top_});
            K::moe_scale_rows(x.x.data, dtype, (const int32_t*)pair_pos.data, (const float*)weight.data, top_, scaled.data, (float*)unit.data, (int)n, (int)hidden_,
                              c.stream);
            first_in = scaled.data;
            first_rows = nullptr;
            sum_weight = (const float*)unit.data;
        }
        if (on_cores) {
            K::moe_product_mfma(first_in, first_rows, gate_up_->t.data, first_stride, act.data, (int)inter_,
                                (int)hidden_, first, gate_.kind, gate_.limit, gate_.alpha, tile_expert, tile_row0, tile_rows,
                                (const int32_t*)n_tiles.data, max_tiles, tile_m, c.stream);
            K::moe_product_mfma(act.data, nullptr, down_->t.data, (long long)(hidden_ * inter_), y.data, (int)hidden_, (int)inter_, 0, 0, 0.f, 1.f,
                                tile_expert, tile_row0, tile_rows, (const int32_t*)n_tiles.data, max_tiles, tile_m, c.stream);
        } else {
            K::moe_product(first_in, dtype, first_rows, gate_up_->t.data, gate_up_->t.dtype, first_stride,
                           act.data, (int)inter_, (int)hidden_, first, gate_.kind, gate_.limit, gate_.alpha, tile_expert, tile_row0, tile_rows,
                           (const int32_t*)n_tiles.data, max_tiles, c.stream);
            K::moe_product(act.data, dtype, nullptr, down_->t.data, down_->t.dtype, (long long)(hidden_ * inter_), y.data, (int)hidden_, (int)inter_, 0,
                           0, 0.f, 1.f, tile_expert, tile_row0, tile_rows, (const int32_t*)n_tiles.data, max_tiles, c.stream);
        }
        Tensor out = c.alloc(dtype, {n, hidden_});
        const float* shared_by = shared_gate_ ? (const float*)shared_scale.data : nullptr;
        // the sum into the stream and the next norm of it in one pass, where that norm is one the kernel knows
        if (stream && next_norm && next_norm->foldable() && next_norm->size() == hidden_ && K::moe_combine_norm_supported.raw((int)hidden_)) {
            const Tensor& w = *next_norm->fold_weight();
            K::moe_combine_norm((float*)stream->h.data, y.data, dtype, (const int32_t*)pair_pos.data, sum_weight, top_, identity_ ? x.x.data : nullptr, shared_out.data,
                                shared_by, beside, scale, w.data, w.dtype, next_norm->fold_eps(), out.data, (int)n, (int)hidden_, c.stream);
            stream->pending = Pending();
            stream->invalidate();
            stream->normed = out;
            stream->normed_for = next_norm;
            return Tensor();
        }
        K::moe_combine(y.data, dtype, (const int32_t*)pair_pos.data, sum_weight, top_, identity_ ? x.x.data : nullptr, shared_out.data,
                       shared_by, beside, scale, out.data, (int)n, (int)hidden_, c.stream);
        return out;
    }

    int64_t hidden_, inter_;
    int n_experts_, top_;
    float router_scale_;
    Gate gate_;
    bool gated_ = true, renormalize_ = false, sigmoid_scores_ = false, weight_on_input_ = false;
    int identity_ = 0, n_groups_ = 1, keep_groups_ = 1;
    bool by_choice_ = false;
    float weight_floor_ = 0.f;
    std::string n_shared_gate_, n_correction_;
    OwnedPtr shared_gate_, correction_, stored_correction_;
    std::string n_router_, n_expert_, n_gate_, n_up_, n_down_, n_shared_;
    std::shared_ptr<FeedForward> shared_;
    OwnedPtr router_, gate_up_, down_;
    Weight w_router_;
};

}  // namespace

void register_moe_parts() {
    register_kind("feed_forward", "routed_experts", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<RoutedExperts>(s, e); });
}

}  // namespace tq
