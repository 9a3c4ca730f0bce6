// Kezasun: a decoder whose layers are listed one by one in its configuration.  A layer is one RMS norm (its weight stored around zero) that a
// mixer and a feed-forward both read, x <- x + m (mixer(h) + ff(h)); the feed-forward may be absent.
// Two mixers.  "wkv": time mixing, a decaying matrix state per head whose inputs mix the token with the one before it.  "attention": grouped-query
// attention over a sliding window with biases, q and k normed over the whole projection, rotation in halves of a head's first elements with
// scaled frequencies, one more 1 in the softmax's denominator (a sink of score 0) and a gate per head; a layer may read an earlier
// layer's keys and values.  The feed-forwards are routed experts chosen by their softmax score plus a correction within the best groups; the
// last of the router's outputs are experts that give back their input.
//
// This file holds what is particular to the architecture: which config.json keys it reads and how they become a ModelSpec with the
// checkpoint's tensor names.  Nothing here computes.
//
// config.json: architecture "Kezasun"; vocab, width; norm.eps; residual_mult; layers: a list of {type, mixer, mlp}.  mixer of "wkv": {heads, dim}; of
// "attention": {heads, kv_heads, dim, vdim, scale, mask {size}, rot {base, dims, scaling {factor, low, high, original} (optional)}, kv_from
// (optional)}.  mlp: null or {kind "moe", expert {ff}, router {experts, top, identity, groups {count, keep}}} (identity 0 and one group unless
// given).  max_positions (optional): the longest sequence, 131072 unless given.
// Tensors: embed, head, final.norm, l<i>.norm1; wkv: l<i>.mix.{mu.r, mu.k, mu.v, mu.g, mu.w, r, k, v, g, w1, w2, w0, u, norm, o}; attention:
// l<i>.mix.{q, q.b, k, k.b, v, v.b, q.norm, k.norm, g, o} (with kv_from no k, v and what belongs to them); l<i>.mlp.{router, correction},
// l<i>.mlp.e<j>.{gate, up, down}.
#include <algorithm>

#include "config.h"

namespace tq {
namespace {

const long long DEFAULT_MAX_POSITIONS = 131072;
const long long DEFAULT_DECAY_RANK = 64;        // what random weights get: the checkpoint's tensors give the rank
const double SINK_SCORE = 0.0;                  // the denominator's extra exp(0): fixed by the design
const double WEIGHT_FLOOR = 1e-20;              // added to the sum the chosen experts' scores are divided by

const Json& object_at(const Json& parent, const char* key, const std::string& where) {
    const Json& j = parent[key];
    if (!j.is_object()) raise(TQE_ERR_CONFIG, "%s: '%s' must be an object", where.c_str(), key);
    return j;
}

Json mixer_typed(const Json& raw, const std::string& where, const std::string& type, const std::vector<Json>& before) {
    KeyReader r(raw, where);
    Json m = Json::object();
    m.set("heads", r.integer("heads", 1));
    m.set("dim", r.integer("dim", 1));
    if (type == "wkv") return m;
    m.set("kv_heads", r.integer("kv_heads", 1));
    m.set("vdim", r.integer("vdim", 1));
    m.set("scale", r.number("scale"));
    m.set("window", KeyReader(object_at(raw, "mask", where), where + ".mask").integer("size", 1));
    if (m["heads"].as_int() % m["kv_heads"].as_int())
        raise(TQE_ERR_CONFIG, "%s: %lld heads are not a multiple of %lld kv_heads", where.c_str(), (long long)m["heads"].as_int(), (long long)m["kv_heads"].as_int());
    KeyReader rot(object_at(raw, "rot", where), where + ".rot");
    const long long dims = rot.integer("dims", 0), dim = m["dim"].as_int();
    if (dims % 2 || dims > dim) raise(TQE_ERR_CONFIG, "%s.rot: dims %lld must be even and at most dim %lld", where.c_str(), dims, dim);
    m.set("rot_base", rot.number("base", true));
    m.set("rot_dims", dims);
    Json scaling;
    if (rot.has("scaling")) {
        KeyReader sc(object_at(rot.raw(), "scaling", where + ".rot"), where + ".rot.scaling");
        scaling = Json::object();
        for (const char* key : {"factor", "low", "high", "original"}) scaling.set(key, sc.number(key, true));
        if (scaling["high"].as_number() <= scaling["low"].as_number())
            raise(TQE_ERR_CONFIG, "%s.rot.scaling: high %g must be more than low %g", where.c_str(), scaling["high"].as_number(), scaling["low"].as_number());
    }
    m.set("rot_scaling", scaling);
    m.set("kv_from", Json());
    if (r.has("kv_from")) {
        const long long from = r.integer("kv_from", 0);
        if (from >= (long long)before.size() || before[(size_t)from]["type"].as_string() != "attention")
            raise(TQE_ERR_CONFIG, "%s: kv_from %lld is no earlier attention layer", where.c_str(), from);
        const Json& lender = before[(size_t)from]["mixer"];
        if (!lender["kv_from"].is_null()) raise(TQE_ERR_CONFIG, "%s: kv_from %lld has no keys and values of its own", where.c_str(), from);
        for (const char* key : {"kv_heads", "dim", "vdim"})
            if (lender[key].as_int() != m[key].as_int())
                raise(TQE_ERR_CONFIG, "%s: its %s %lld is not layer %lld's (%lld), whose keys and values it reads", where.c_str(), key, (long long)m[key].as_int(), from,
                      (long long)lender[key].as_int());
        m.set("kv_from", from);
    }
    return m;
}

Json mlp_typed(const Json& raw, const std::string& where) {
    if (raw.is_null()) return Json();
    if (!raw.is_object()) raise(TQE_ERR_CONFIG, "%s must be an object or null", where.c_str());
    const std::string kind = KeyReader(raw, where).string("kind");
    if (kind != "moe") raise(TQE_ERR_CONFIG, "%s: unknown kind '%s' (known: moe)", where.c_str(), kind.c_str());
    Json m = Json::object();
    m.set("kind", kind);
    m.set("ff", KeyReader(object_at(raw, "expert", where), where + ".expert").integer("ff", 1));
    const std::string rw = where + ".router";
    KeyReader router(object_at(raw, "router", where), rw);
    m.set("experts", router.integer("experts", 1));
    m.set("top", router.integer("top", 1));
    m.set("identity", router.integer_or("identity", 0, 0));
    long long count = 1, keep = 1;
    if (router.has("groups")) {
        KeyReader groups(object_at(router.raw(), "groups", rw), rw + ".groups");
        count = groups.integer("count", 1);
        keep = groups.integer("keep", 1);
    }
    m.set("groups", count);
    m.set("keep", keep);
    const long long outputs = m["experts"].as_int() + m["identity"].as_int();
    if (outputs % count) raise(TQE_ERR_CONFIG, "%s.groups: count %lld does not divide the %lld experts", rw.c_str(), count, outputs);
    if (keep > count) raise(TQE_ERR_CONFIG, "%s.groups: keep %lld of %lld groups", rw.c_str(), keep, count);
    if (m["top"].as_int() > keep * (outputs / count))
        raise(TQE_ERR_CONFIG, "%s: top %lld of the %lld experts that the groups kept hold", rw.c_str(), (long long)m["top"].as_int(), keep * (outputs / count));
    return m;
}

Json kezasun_typed(const Json& raw, const std::string& where) {
    KeyReader r(raw, where);
    Json c = Json::object();
    c.set("vocab", r.integer("vocab", 1));
    c.set("width", r.integer("width", 1));
    c.set("norm_eps", KeyReader(object_at(raw, "norm", where), where + ": norm").number("eps"));
    c.set("residual_mult", r.number("residual_mult"));
    c.set("max_positions", r.integer_or("max_positions", DEFAULT_MAX_POSITIONS, 1));
    if (!raw["layers"].is_array() || raw["layers"].items().empty()) raise(TQE_ERR_CONFIG, "%s: 'layers' must be a list of at least one layer", where.c_str());
    std::vector<Json> typed;
    Json list = Json::array();
    for (const Json& l : raw["layers"].items()) {
        const std::string at = format("%s: layers[%zu]", where.c_str(), typed.size());
        if (!l.is_object()) raise(TQE_ERR_CONFIG, "%s must be an object", at.c_str());
        const std::string type = KeyReader(l, at).string("type");
        if (type != "wkv" && type != "attention") raise(TQE_ERR_CONFIG, "%s: unknown type '%s' (known: attention, wkv)", at.c_str(), type.c_str());
        Json t = Json::object();
        t.set("type", type);
        t.set("mixer", mixer_typed(object_at(l, "mixer", at), at + ".mixer", type, typed));
        t.set("mlp", mlp_typed(l["mlp"], at + ".mlp"));
        typed.push_back(t);
        list.push(t);
    }
    c.set("layers", list);
    return c;
}

PartSpec part(const char* kind, std::initializer_list<std::pair<const char*, Json>> params) {
    PartSpec p;
    p.kind = kind;
    for (const auto& kv : params) p.params.set(kv.first, kv.second);
    return p;
}

Json names_of(std::initializer_list<std::pair<const char*, const char*>> pairs) {
    Json n = Json::object();
    for (const auto& kv : pairs) n.set(kv.first, kv.second);
    return n;
}

ModelSpec kezasun_spec(const Json& c) {
    const long long width = c["width"].as_int();
    const Json& eps = c["norm_eps"];
    const Json& max_pos = c["max_positions"];
    const std::vector<Json>& layers = c["layers"].items();
    const PartSpec norm = part("rms_norm", {{"size", width}, {"eps", eps}, {"unit_offset", true}, {"tensor", ""}});
    // What a layer's cache keeps: the largest window of the layers that read it.  Equal pages with equal windows are one group of the cache, and the
    // cache's bookkeeping takes TQE_MAX_GROUPS of them: with more, layers of equal pages keep the largest of their windows.
    auto is_attention = [&](size_t l) { return layers[l]["type"].as_string() == "attention"; };
    auto owner_of = [&](size_t l) { const Json& from = layers[l]["mixer"]["kv_from"]; return from.is_null() ? l : (size_t)from.as_int(); };
    auto pages_of = [&](size_t l) { const Json& m = layers[l]["mixer"]; return std::vector<long long>{m["kv_heads"].as_int(), m["dim"].as_int(), m["vdim"].as_int()}; };
    std::vector<long long> keep(layers.size(), 0);
    for (size_t l = 0; l < layers.size(); ++l)
        if (is_attention(l)) keep[owner_of(l)] = std::max(keep[owner_of(l)], (long long)layers[l]["mixer"]["window"].as_int());
    std::vector<std::vector<long long>> distinct;
    for (size_t l = 0; l < layers.size(); ++l) {
        if (!is_attention(l) || owner_of(l) != l) continue;
        std::vector<long long> key = pages_of(l);
        key.push_back(keep[l]);
        if (std::find(distinct.begin(), distinct.end(), key) == distinct.end()) distinct.push_back(key);
    }
    if ((int)distinct.size() > TQE_MAX_GROUPS) {
        const std::vector<long long> own = keep;
        for (size_t l = 0; l < layers.size(); ++l)
            for (size_t o = 0; o < layers.size(); ++o)
                if (is_attention(l) && is_attention(o) && owner_of(l) == l && owner_of(o) == o && pages_of(l) == pages_of(o)) keep[l] = std::max(keep[l], own[o]);
    }
    ModelSpec s;
    s.architecture = "Kezasun";
    s.vocab_size = c["vocab"].as_int();
    s.hidden_size = width;
    s.max_positions = c["max_positions"].as_int();
    s.embedding_name = "embed";
    for (size_t l = 0; l < layers.size(); ++l) {
        const Json& m = layers[l]["mixer"];
        const Json& mlp = layers[l]["mlp"];
        PartSpec mixer;
        Run run;
        run.layer = (int)l;
        if (is_attention(l)) {
            const bool own = m["kv_from"].is_null();
            PartSpec position = part("none", {{"max_positions", max_pos}});
            if (m["rot_dims"].as_int() > 0) {
                position = part("rotary", {{"theta", m["rot_base"]}, {"rot_dim", m["rot_dims"]}, {"max_positions", max_pos}, {"style", "halves"}});
                if (!m["rot_scaling"].is_null()) position.params.set("scaling", m["rot_scaling"]);
            }
            mixer = part("attention", {{"hidden", width}, {"n_heads", m["heads"]}, {"n_kv_heads", m["kv_heads"]}, {"head_dim", m["dim"]}, {"value_dim", m["vdim"]},
                {"scale", m["scale"]}, {"qkv_bias", true}, {"qk_norm", true}, {"qk_norm_over", "projection"}, {"eps", eps}, {"window", m["window"]},
                {"cache_window", keep[owner_of(l)]}, {"sink_score", SINK_SCORE}, {"gate", "head"}, {"own_kv", own}, {"position", position.to_json()},
                {"names", names_of({{"q", "q"}, {"k", "k"}, {"v", "v"}, {"o", "o"}, {"q_norm", "q.norm"}, {"k_norm", "k.norm"}, {"gate", "g"}, {"q_bias", "q.b"},
                                    {"k_bias", "k.b"}, {"v_bias", "v.b"}})}});
            if (!own) run.cache_of = (int)m["kv_from"].as_int();
        } else {
            mixer = part("time_mixing", {{"hidden", width}, {"heads", m["heads"]}, {"head_dim", m["dim"]}, {"decay_rank", DEFAULT_DECAY_RANK}, {"eps", eps},
                {"names", names_of({{"mu", "mu."}, {"r", "r"}, {"k", "k"}, {"v", "v"}, {"g", "g"}, {"o", "o"}, {"w1", "w1"}, {"w2", "w2"}, {"w0", "w0"}, {"bonus", "u"},
                                    {"norm", "norm"}})}});
        }
        Json ff;
        if (!mlp.is_null())
            ff = part("routed_experts", {{"hidden", width}, {"inter", mlp["ff"]}, {"n_experts", mlp["experts"]}, {"top", mlp["top"]}, {"router_scale", 1.0},
                {"gate", "silu"}, {"normalize", "chosen"}, {"identity", mlp["identity"]}, {"correction", "correction"}, {"n_groups", mlp["groups"]},
                {"keep_groups", mlp["keep"]}, {"weight_floor", WEIGHT_FLOOR}, {"shared", Json()},
                {"names", names_of({{"router", "router"}, {"expert", "e%d."}, {"gate", "gate"}, {"up", "up"}, {"down", "down"}})}}).to_json();
        LayerSpec spec;
        spec.prefix = format("l%zu.", l);
        spec.block = part("joint", {{"mixer", mixer.to_json()}, {"feed_forward", ff}, {"norm", norm.to_json()}, {"scale", c["residual_mult"]},
            {"names", names_of({{"mixer", "mix."}, {"feed_forward", "mlp."}, {"norm", "norm1"}})}});
        s.layers.push_back(spec);
        s.order.push_back(run);
    }
    s.final_norm = norm;
    s.final_norm_prefix = "final.norm";
    s.head_name = "head";
    return s;
}

}  // namespace

void register_kezasun() {
    Architecture a;
    a.name = "Kezasun";
    a.model_types = {"kezasun"};
    a.typed_config = kezasun_typed;
    a.build_spec = kezasun_spec;
    register_architecture(a);
}

}  // namespace tq
