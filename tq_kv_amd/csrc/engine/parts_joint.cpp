// A block whose mixer and feed-forward run side by side on one norm of the stream.
//
//   block joint   h = norm(x), x' = x + scale (mixer(h) + ff(h)); the feed-forward may be absent.
//
// The sum is formed in the feed-forward's own last kernel where it offers that (takes_beside), which may also add it to the stream and work out the
// next block's norm; else it is left pending on the stream for the next norm's kernel.
//
// params: mixer, feed_forward (or null), norm (part specs), scale (1 unless given); names {mixer, feed_forward, norm}: prefixes of the parts' tensors.
#include "kernels.h"
#include "linear.h"
#include "parts.h"
#include "step.h"
#include "trace.h"

namespace tq {
namespace {

class JointBlock : public Block {
public:
    JointBlock(const PartSpec& spec, BuildEnv& env) {
        KeyReader r(spec.params, "joint block", TQE_ERR_ARGUMENT);
        scale_ = (float)r.number_or("scale", 1.0);
        const Json& names = spec.params["names"];
        auto one = [&](const char* role, const char* category, bool optional) -> std::shared_ptr<Part> {
            const Json& p = spec.params[role];
            if (p.is_null()) {
                if (optional) return nullptr;
                raise(TQE_ERR_ARGUMENT, "joint block: no '%s' given", role);
            }
            std::shared_ptr<Part> part = build_part(category, PartSpec::from_json(p, role), env);
            if (!names[role].is_string()) raise(TQE_ERR_ARGUMENT, "joint block: no tensor-name prefix for '%s'", role);
            roles_.push_back({role, names[role].as_string(), part});
            return part;
        };
        mixer_ = std::dynamic_pointer_cast<Mixer>(one("mixer", "mixer", false));
        feed_forward_ = std::dynamic_pointer_cast<FeedForward>(one("feed_forward", "feed_forward", true));
        norm_ = std::dynamic_pointer_cast<Norm>(one("norm", "norm", false));
        if (!mixer_ || !norm_ || (!feed_forward_ && !spec.params["feed_forward"].is_null())) raise(TQE_ERR_ARGUMENT, "joint block: a part is of the wrong category");
        graph_safe = true;
        for (const Role& role : roles_) graph_safe = graph_safe && role.part->graph_safe;
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
            for (const auto& t : r.part->tensors()) {
                auto it = tensors.find(r.prefix + t.first);
                if (it == tensors.end() || !it->second) raise(TQE_ERR_WEIGHTS, "a part was not given its tensor '%s'", (r.prefix + t.first).c_str());
                own[t.first] = it->second;
            }
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
    Norm* first_norm() override { return norm_.get(); }
    Mixer* mixer() override { return mixer_.get(); }

    Stream* forward(StepContext& c, Stream* stream, const CacheEntry& entry, Norm* next_norm, bool last) override {
        // the model's last block goes on with the wanted rows alone: keys and values of all tokens, everything else of those rows
        const bool prune = last && c.prune_last && policy().prune_last && mixer_->takes_rows;
        Activation x;
        if (stream->normed_for == norm_.get() && stream->pending.kind == Pending::Nothing && stream->normed.dtype == c.act_dtype) {
            x.x = stream->normed;
            stream->invalidate();
        } else {
            Span span(norm_->trace_name());
            x.x = c.alloc(c.act_dtype, {stream->h.shape[0], stream->h.shape[1]});
            norm_->add_norm(c, stream->h, stream->pending, x.x);
            stream->pending = Pending();
            stream->invalidate();
        }
        Tensor y;
        {
            Span span(mixer_->trace_name());
            y = mixer_->forward(c, x, entry, nullptr, prune);
        }
        if (prune) {
            c.sub_stream.reset(new Stream());
            Stream* sub = c.sub_stream.get();
            sub->of_last_rows = true;
            sub->h = c.alloc(F32, {c.n_last, stream->h.shape[1]});
            if (c.n_last == 0) return sub;
            k_gather_rows(c, stream->h, c.dev.last_rows, c.n_last, sub->h);
            if (feed_forward_) {
                Tensor rows = c.alloc(x.x.dtype, {c.n_last, x.x.shape[1]});
                k_gather_rows(c, x.x, c.dev.last_rows, c.n_last, rows);
                x.x = rows;
            }
            stream = sub;
        }
        Tensor out;
        if (feed_forward_ && feed_forward_->takes_beside()) {
            Span span(feed_forward_->trace_name());
            // (what the head reads after the last block is chosen rows: their norm is the head's)
            out = feed_forward_->forward_beside(c, x, y, scale_, last ? nullptr : stream, last ? nullptr : next_norm);
            if (!out.defined()) return stream;
        } else {
            Tensor f;
            if (feed_forward_) {
                Span span(feed_forward_->trace_name());
                f = feed_forward_->forward(c, x, nullptr);
            }
            out = c.alloc(y.dtype, {y.shape[0], y.shape[1]});
            K::scaled_sum(y.data, f.data, y.dtype, scale_, out.data, (long long)y.numel(), c.stream);
        }
        stream->pending = Pending::of(out);
        stream->invalidate();
        return stream;
    }

private:
    struct Role { std::string role, prefix; std::shared_ptr<Part> part; };
    float scale_ = 1.f;
    std::vector<Role> roles_;
    std::shared_ptr<Mixer> mixer_;
    std::shared_ptr<FeedForward> feed_forward_;
    std::shared_ptr<Norm> norm_;
};

}  // namespace

void register_joint_parts() {
    register_kind("block", "joint", [](const PartSpec& s, BuildEnv& e) { return std::make_shared<JointBlock>(s, e); });
}

}  // namespace tq
