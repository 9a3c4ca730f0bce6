// Rasodra: a decoder whose layers are listed one by one in its configuration.  A sublayer has a norm on both sides, x <- x + N_b(part(N_a(x)))
// with layer norms that have a weight and no bias; a layer is a mixer and an optional feed-forward, down(max(up, 0)^2).  A layer may name
// another layer whose tensors it uses: then it runs with that layer's weights, with a cache or state of its own.
// Three mixers.  "mlstm": a matrix memory with gates kept as logarithms against a running maximum.  "latent_attention": attention through
// one cached latent and one rotated key part per position, queries straight from the input, a sink, an output gate for every element.
// "attention": grouped-query attention with biases whose values are its keys as projected, heads normed with a weight in front of a rotation by
// neighbouring pairs, positions in chunks that see nothing of an earlier chunk.
//
// This file holds what is particular to the architecture: which config.json keys it reads and how they become a ModelSpec with the
// checkpoint's tensor names.  Nothing here computes.
//
// config.json: architecture "Rasodra"; vocab, width; norm.eps; layers: a list of {type, mixer, mlp, weights_of (optional)}.  mixer of "mlstm":
// {heads, dim, vdim, gate_cap}; of "latent_attention": {heads, dim, rot_dim, vdim, kv_rank, scale, rot {base, dims}}; of "attention": {heads,
// kv_heads, dim, vdim, scale, mask {size}, rot {base, dims}}.  mlp: null or {kind "dense", ff}.  max_positions (optional): the longest sequence,
// 131072 unless given.
// Tensors: embed, head, final.norm, l<i>.norm1, l<i>.norm1b, l<i>.norm2, l<i>.norm2b; mlstm: l<i>.mix.{q, k, v, g, o, norm, i, i.b, f, f.b};
// latent_attention: l<i>.mix.{q, dkv, dkv.norm, uk, uv, sink, g, o}; attention: l<i>.mix.{q, q.b, k, k.b, q.norm, k.norm, o}; l<i>.mlp.{up, down}.
#include <set>

#include "config.h"

namespace tq {
namespace {

const long long DEFAULT_MAX_POSITIONS = 131072;

const Json& object_at(const Json& parent, const char* key, const std::string& where) {
    const Json& j = parent[key];
    if (!j.is_object()) raise(TQE_ERR_CONFIG, "%s: '%s' must be an object", where.c_str(), key);
    return j;
}

void rot_typed(const Json& raw, const std::string& where, long long most, const char* what, Json& m) {
    KeyReader rot(object_at(raw, "rot", where), where + ".rot");
    const long long dims = rot.integer("dims", 0);
    if (dims % 2 || dims > most) raise(TQE_ERR_CONFIG, "%s.rot: dims %lld must be even and at most %s %lld", where.c_str(), dims, what, most);
    m.set("rot_base", rot.number("base", true));
    m.set("rot_dims", dims);
}

Json mixer_typed(const Json& raw, const std::string& where, const std::string& type) {
    KeyReader r(raw, where);
    Json m = Json::object();
    m.set("heads", r.integer("heads", 1));
    m.set("dim", r.integer("dim", 1));
    m.set("vdim", r.integer("vdim", 1));
    if (type == "mlstm") {
        m.set("gate_cap", r.number("gate_cap", true));
    } else if (type == "latent_attention") {
        m.set("rot_dim", r.integer("rot_dim", 0));
        m.set("kv_rank", r.integer("kv_rank", 1));
        m.set("scale", r.number("scale", true));
        rot_typed(raw, where, m["rot_dim"].as_int(), "rot_dim", m);
    } else {
        m.set("kv_heads", r.integer("kv_heads", 1));
        m.set("scale", r.number("scale", true));
        m.set("chunk", KeyReader(object_at(raw, "mask", where), where + ".mask").integer("size", 1));
        if (m["heads"].as_int() % m["kv_heads"].as_int())
            raise(TQE_ERR_CONFIG, "%s: %lld heads are not a multiple of %lld kv_heads", where.c_str(), (long long)m["heads"].as_int(), (long long)m["kv_heads"].as_int());
        if (m["dim"].as_int() != m["vdim"].as_int())
            raise(TQE_ERR_CONFIG, "%s: the values are the keys, so vdim %lld must be dim %lld", where.c_str(), (long long)m["vdim"].as_int(), (long long)m["dim"].as_int());
        rot_typed(raw, where, m["dim"].as_int(), "dim", m);
    }
    return m;
}

Json mlp_typed(const Json& raw, const std::string& where) {
    if (raw.is_null()) return Json();
    if (!raw.is_object()) raise(TQE_ERR_CONFIG, "%s must be an object or null", where.c_str());
    KeyReader r(raw, where);
    const std::string kind = r.string("kind");
    if (kind != "dense") raise(TQE_ERR_CONFIG, "%s: unknown kind '%s' (known: dense)", where.c_str(), kind.c_str());
    Json m = Json::object();
    m.set("kind", kind);
    m.set("ff", r.integer("ff", 1));
    return m;
}

Json rasodra_typed(const Json& raw, const std::string& where) {
    KeyReader r(raw, where);
    Json c = Json::object();
    c.set("vocab", r.integer("vocab", 1));
    c.set("width", r.integer("width", 1));
    c.set("norm_eps", KeyReader(object_at(raw, "norm", where), where + ": norm").number("eps"));
    c.set("max_positions", r.integer_or("max_positions", DEFAULT_MAX_POSITIONS, 1));
    if (!raw["layers"].is_array() || raw["layers"].items().empty()) raise(TQE_ERR_CONFIG, "%s: 'layers' must be a list of at least one layer", where.c_str());
    Json list = Json::array();
    std::vector<Json> typed;
    for (const Json& l : raw["layers"].items()) {
        const long long i = (long long)typed.size();
        const std::string at = format("%s: layers[%lld]", where.c_str(), i);
        if (!l.is_object()) raise(TQE_ERR_CONFIG, "%s must be an object", at.c_str());
        KeyReader lr(l, at);
        const std::string type = lr.string("type");
        if (type != "mlstm" && type != "latent_attention" && type != "attention")
            raise(TQE_ERR_CONFIG, "%s: unknown type '%s' (known: attention, latent_attention, mlstm)", at.c_str(), type.c_str());
        Json t = Json::object();
        t.set("type", type);
        t.set("mixer", mixer_typed(object_at(l, "mixer", at), at + ".mixer", type));
        t.set("mlp", mlp_typed(l["mlp"], at + ".mlp"));
        t.set("source", lr.has("weights_of") ? lr.integer("weights_of", 0) : i);
        typed.push_back(t);
    }
    // whose tensors a layer uses: its own, or those of another layer of the same sizes (which may itself use another's)
    const long long n = (long long)typed.size();
    for (long long i = 0; i < n; ++i) {
        const std::string at = format("%s: layers[%lld]", where.c_str(), i);
        long long source = i;
        for (long long steps = 0; source >= n || typed[(size_t)source]["source"].as_int() != source; ++steps) {
            if (source >= n || steps == n) raise(TQE_ERR_CONFIG, "%s: weights_of leads to no layer with tensors of its own", at.c_str());
            source = typed[(size_t)source]["source"].as_int();
        }
        Json t = typed[(size_t)i];
        for (const char* key : {"type", "mixer", "mlp"})
            if (t[key].dump() != typed[(size_t)source][key].dump())
                raise(TQE_ERR_CONFIG, "%s: its %s is not that of layer %lld, whose tensors it uses", at.c_str(), key, source);
        t.set("source", source);
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

ModelSpec rasodra_spec(const Json& c) {
    const long long width = c["width"].as_int();
    const Json& eps = c["norm_eps"];
    const Json& max_pos = c["max_positions"];
    const Json norm = part("layer_norm", {{"size", width}, {"eps", eps}, {"tensor", ""}, {"bias", false}}).to_json();
    auto rotary = [&](const Json& m) {
        if (m["rot_dims"].as_int() == 0) return part("none", {{"max_positions", max_pos}}).to_json();
        return part("rotary", {{"theta", m["rot_base"]}, {"rot_dim", m["rot_dims"]}, {"max_positions", max_pos}, {"style", "pairs"}}).to_json();
    };
    ModelSpec s;
    s.architecture = "Rasodra";
    s.vocab_size = c["vocab"].as_int();
    s.hidden_size = width;
    s.max_positions = c["max_positions"].as_int();
    s.embedding_name = "embed";
    // Every kind of page and every size of chunk is a group of the cache, and the cache's bookkeeping takes TQE_MAX_GROUPS of them: with
    // more, the chunked layers keep every page, so that those with equal pages share one group.
    std::set<std::string> groups;
    for (const Json& layer : c["layers"].items()) {
        const Json& m = layer["mixer"];
        if (layer["type"].as_string() == "latent_attention") groups.insert(format("l %lld %lld", (long long)m["kv_rank"].as_int(), (long long)m["rot_dim"].as_int()));
        if (layer["type"].as_string() == "attention")
            groups.insert(format("a %lld %lld %lld", (long long)m["kv_heads"].as_int(), (long long)m["dim"].as_int(), (long long)m["chunk"].as_int()));
    }
    const bool keep_all = (int)groups.size() > TQE_MAX_GROUPS;
    std::map<long long, int> index;                     // layers with tensors of their own, by their number in the list
    long long number = 0;
    for (const Json& layer : c["layers"].items()) {
        const Json& m = layer["mixer"];
        const Json& mlp = layer["mlp"];
        if (layer["source"].as_int() == number) {
            const std::string type = layer["type"].as_string();
            PartSpec mixer;
            if (type == "mlstm")
                mixer = part("mlstm", {{"hidden", width}, {"heads", m["heads"]}, {"head_dim", m["dim"]}, {"value_dim", m["vdim"]}, {"gate_cap", m["gate_cap"]}, {"eps", eps},
                    {"names", names_of({{"q", "q"}, {"k", "k"}, {"v", "v"}, {"g", "g"}, {"o", "o"}, {"norm", "norm"}, {"i", "i"}, {"i_bias", "i.b"}, {"f", "f"}, {"f_bias", "f.b"}})}});
            else if (type == "latent_attention")
                mixer = part("latent_attention", {{"hidden", width}, {"n_heads", m["heads"]}, {"head_dim", m["dim"]}, {"rot_dim", m["rot_dim"]}, {"value_dim", m["vdim"]},
                    {"q_rank", Json()}, {"kv_rank", m["kv_rank"]}, {"scale", m["scale"]}, {"eps", eps}, {"window", Json()}, {"cache_window", Json()}, {"own_kv", true},
                    {"gate", true}, {"gate_per", "element"}, {"sink", true}, {"position", rotary(m)}});
            else
                mixer = part("attention", {{"hidden", width}, {"n_heads", m["heads"]}, {"n_kv_heads", m["kv_heads"]}, {"head_dim", m["dim"]}, {"values_are_keys", true},
                    {"scale", m["scale"]}, {"qkv_bias", true}, {"qk_norm", true}, {"eps", eps}, {"chunk", m["chunk"]}, {"cache_keeps_all", keep_all}, {"position", rotary(m)},
                    {"names", names_of({{"q", "q"}, {"k", "k"}, {"o", "o"}, {"q_norm", "q.norm"}, {"k_norm", "k.norm"}, {"q_bias", "q.b"}, {"k_bias", "k.b"}})}});
            Json ff;
            if (!mlp.is_null())
                ff = part("activated", {{"hidden", width}, {"inter", mlp["ff"]}, {"gate", "relu2"}, {"names", names_of({{"up", "up"}, {"down", "down"}})}}).to_json();
            LayerSpec spec;
            spec.prefix = format("l%lld.", number);
            spec.block = part("pre_norm", {{"mixer", mixer.to_json()}, {"feed_forward", ff}, {"mixer_norm", norm}, {"ff_norm", mlp.is_null() ? Json() : norm},
                {"post_mixer_norm", norm}, {"post_ff_norm", mlp.is_null() ? Json() : norm},
                {"names", names_of({{"mixer", "mix."}, {"feed_forward", "mlp."}, {"mixer_norm", "norm1"}, {"ff_norm", "norm2"}, {"post_mixer_norm", "norm1b"},
                                    {"post_ff_norm", "norm2b"}})}});
            index[number] = (int)s.layers.size();
            s.layers.push_back(spec);
        }
        ++number;
    }
    for (const Json& layer : c["layers"].items()) {
        Run run;
        run.layer = index.at(layer["source"].as_int());
        s.order.push_back(run);
    }
    s.final_norm = PartSpec::from_json(norm, "final norm");
    s.final_norm_prefix = "final.norm";
    s.head_name = "head";
    return s;
}

}  // namespace

void register_rasodra() {
    Architecture a;
    a.name = "Rasodra";
    a.model_types = {"rasodra"};
    a.typed_config = rasodra_typed;
    a.build_spec = rasodra_spec;
    register_architecture(a);
}

}  // namespace tq
