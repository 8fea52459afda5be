// vuzazen.cc — loading a Vuzazen folder (novorax.h describes the design, config_model.h the shared loader).
//
// A layer is x += mixer(norm(x)), then x += ff(norm(x)): norms in front of the sublayers only, so the last product of a sublayer adds into the stream itself
// (nvx_close_linear) and no launch stands between two sublayers.  Every mixer is one the folder designs share - the mLSTM and the latent attention of
// novorax.cc (the latter with halves turning and an output gate per head, its gate rows riding in the down-projection), the grouped-query attention of
// fidepel.cc (with the short convolution, unit values and mixed scores switched on) - and so is the feed-forward: dense silu, or the routed experts whose
// weight multiplies what the expert reads.
#include <cmath>

#include "config_model.h"

namespace mi355 {

Model *vuzazen_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status) {
    (void)dir;
    status = -102;
    Model *const m = ld.m;
    NovoraxModel &M = *m->nvx;
    M.design = "vuzazen";
    M.norm_off = 1.0f;
    const int W = (int)cfg["width"].as_int(), V = (int)cfg["vocab"].as_int();
    if (!cfg_positive(err, "width", W) || !cfg_positive(err, "vocab", V)) return nullptr;
    M.width = W; M.n_vocab = V;
    M.eps = (float)cfg["norm"]["eps"].as_double(1e-6);
    const Json &em = cfg["embedding"];
    M.embed_scale = (float)em["scale"].as_double(1.0);
    const Json &layers = cfg["layers"];
    if (!layers.is_array() || layers.size() == 0 || layers.size() > 1024) { err = "configuration: 'layers' must list 1 .. 1024 layers"; return nullptr; }
    const int nl = (int)layers.size();

    M.embed = ld.embedding("embed", V, W);                      // the table the tokens' rows come from ...
    M.head = ld.rows({{"embed", V}}, W);                        // ... is the output head too (dense rows for the linear kernels)
    M.final_norm = ld.vec("final.norm", W);
    const Json &bg = em["bigram"];
    if (bg.is_object()) {
        const int64_t buckets = bg["buckets"].as_int();
        if (!cfg_positive(err, "embedding.bigram.buckets", buckets)) return nullptr;
        M.bigram_buckets = (int)buckets; M.bigram_mul_prev = bg["mul_prev"].as_int(); M.bigram_mul_cur = bg["mul_cur"].as_int();
        if (M.bigram_mul_prev < 0 || M.bigram_mul_cur < 0 || M.bigram_mul_prev > (1ll << 31) || M.bigram_mul_cur > (1ll << 31)) { err = "configuration: embedding.bigram multipliers are out of range"; return nullptr; }
        M.bigram = ld.embedding("bigram", M.bigram_buckets + 1, W);
    }
    uint64_t active_bytes = ((uint64_t)V * W + 2 * (uint64_t)W) * 2;   // what one token reads of the weights: the head and two table rows, then every layer's matrices

    M.layers.resize((size_t)nl);
    for (int il = 0; il < nl && ld.err.empty(); il++) {
        const Json &lc = layers.at((size_t)il), &mx = lc["mixer"];
        NvxLayer &L = M.layers[(size_t)il];
        const std::string p = "l" + std::to_string(il) + ".", pm = p + "mix.";
        const std::string type = lc["type"].as_string();
        const std::string at = "configuration: layer " + std::to_string(il) + ": ";
        L.norm1 = ld.vec(p + "norm1", W);
        L.heads = (int)mx["heads"].as_int(); L.kv_heads = (int)mx["kv_heads"].as_int(L.heads); L.dim = (int)mx["dim"].as_int(); L.vdim = (int)mx["vdim"].as_int(L.dim);
        if (!cfg_positive(err, "mixer.heads", L.heads, 4096) || !cfg_positive(err, "mixer.kv_heads", L.kv_heads, L.heads) || !cfg_positive(err, "mixer.dim", L.dim, 1 << 16) ||
            !cfg_positive(err, "mixer.vdim", L.vdim, 1 << 16)) return nullptr;
        if (L.heads % L.kv_heads != 0) { err = at + "mixer.heads must be a multiple of mixer.kv_heads"; return nullptr; }
        const int H = L.heads, G = L.kv_heads, D = L.dim, VD = L.vdim;
        if (type == "mlstm") {
            L.type = NVX_MLSTM;
            L.gate_cap = (float)mx["gate_cap"].as_double(0.0);
            if (!(L.gate_cap > 0.0f)) { err = at + "mixer.gate_cap must be positive"; return nullptr; }
            if (!mlstm_shape_ok(D, VD)) { err = "mlstm: dim " + std::to_string(D) + " is beyond what the recurrence kernel keeps in registers (512)"; return nullptr; }
            L.proj = ld.rows({{pm + "q", H * D}, {pm + "k", H * D}, {pm + "v", H * VD}, {pm + "g", H * VD}, {pm + "i", H}, {pm + "f", H}}, W);
            L.i_bias = ld.vec(pm + "i.b", H);
            L.f_bias = ld.vec(pm + "f.b", H);
            L.mix_norm = ld.vec(pm + "norm", H * VD);
            M.max_mlstm_heads = std::max(M.max_mlstm_heads, H);
            M.max_proj = std::max(M.max_proj, L.proj.N);
            active_bytes += (uint64_t)L.proj.N * W * 2;
        } else if (type == "latent_attention") {
            L.type = NVX_LATENT;
            L.rot = (int)mx["rot_dim"].as_int(0); L.kv_rank = (int)mx["kv_rank"].as_int(); L.q_rank = (int)mx["q_rank"].as_int();
            if (!cfg_positive(err, "mixer.kv_rank", L.kv_rank) || !cfg_positive(err, "mixer.q_rank", L.q_rank)) return nullptr;
            if (L.rot < 0 || (L.rot & 1)) { err = at + "mixer.rot_dim must be even and not negative"; return nullptr; }
            if (!latent_attn_shape_ok(L.kv_rank, L.rot)) { err = "latent attention: kv_rank " + std::to_string(L.kv_rank) + " (+ rot_dim) is beyond what the attention kernel holds per lane (1088)"; return nullptr; }
            L.scale = (float)mx["scale"].as_double(1.0);
            L.rot_dims = L.rot;                                  // the whole shared part turns
            L.rot_halves = true;
            const double base = mx["rot"]["base"].as_double(10000.0);
            if (!(base > 0.0)) { err = at + "rot.base must be positive"; return nullptr; }
            L.rot_freq = ld.rot_table(base, L.rot_dims, Json(), nullptr);
            const int QD = D + L.rot;
            L.down = ld.rows({{pm + "dq", L.q_rank}, {pm + "dkv", L.kv_rank + L.rot}, {pm + "g", H}}, W);
            L.off_gate = L.q_rank + L.kv_rank + L.rot;
            L.dq_norm = ld.vec(pm + "dq.norm", L.q_rank);
            L.dkv_norm = ld.vec(pm + "dkv.norm", L.kv_rank);
            L.uq = ld.rows({{pm + "uq", H * QD}}, L.q_rank);
            L.uk_t = ld.head_transposed(pm + "uk", H, D, L.kv_rank);
            L.uv = ld.rows({{pm + "uv", H * VD}}, L.kv_rank);
            M.max_down = std::max(M.max_down, L.down.N);
            M.max_q_rank = std::max(M.max_q_rank, L.q_rank);
            M.max_q = std::max(M.max_q, H * QD);
            M.max_qa = std::max(M.max_qa, H * L.kv_rank);
            active_bytes += ((uint64_t)L.down.N * W + (uint64_t)H * QD * L.q_rank + (uint64_t)H * (D + VD) * L.kv_rank) * 2;
        } else if (type == "attention") {
            L.type = NVX_GQ;
            if (!talk_attn_shape_ok(H, G, D, VD)) {
                err = "attention: heads " + std::to_string(H) + " x (dim " + std::to_string(D) + ", vdim " + std::to_string(VD) + ") are beyond what the attention kernel holds (dim, vdim 512; all heads' rows in LDS)";
                return nullptr;
            }
            L.scale = (float)mx["scale"].as_double(1.0);
            const int NQ = H * D, NK = G * D, NV = G * VD;
            L.off_gate = NQ + NK + NV;
            L.proj = ld.rows({{pm + "q", NQ}, {pm + "k", NK}, {pm + "v", NV}, {pm + "g", H}}, W);
            L.conv_taps = (int)mx["conv"].as_int(1);
            if (!cfg_positive(err, "mixer.conv", L.conv_taps, 64)) return nullptr;
            if (L.off_gate > GQ_CONV_MAX_CHANNELS) { err = at + "q, k and v have more rows than the convolution holds (" + std::to_string(GQ_CONV_MAX_CHANNELS) + ")"; return nullptr; }
            L.conv_wt = ld.rows_f32_transposed({{pm + "q.conv", NQ}, {pm + "k.conv", NK}, {pm + "v.conv", NV}}, L.conv_taps);
            L.q_norm = ld.vec(pm + "q.norm", NQ);
            L.k_norm = ld.vec(pm + "k.norm", NK);
            L.v_unit = true;
            L.talk = ld.rows_f32({{pm + "talk", H}}, H);
            M.max_proj = std::max(M.max_proj, L.proj.N);
            M.max_q = std::max(M.max_q, NQ);
            active_bytes += (uint64_t)L.proj.N * W * 2;
        } else { err = at + "unknown type '" + type + "'"; return nullptr; }
        L.o = ld.rows({{pm + "o", W}}, H * VD);
        M.max_att = std::max(M.max_att, H * VD);
        active_bytes += (uint64_t)W * H * VD * 2;

        const Json &mlp = lc["mlp"];
        if (mlp.is_object()) {
            const std::string pf = p + "mlp.";
            const std::string kind = mlp["kind"].as_string();
            L.norm2 = ld.vec(p + "norm2", W);
            if (kind == "dense") {
                L.ff_kind = NVX_FF_DENSE;
                L.ff = (int)mlp["ff"].as_int();
                if (!cfg_positive(err, "mlp.ff", L.ff)) return nullptr;
                L.gate = ld.rows({{pf + "gate", L.ff}}, W);
                L.up = ld.rows({{pf + "up", L.ff}}, W);
                L.down_ff = ld.rows({{pf + "down", W}}, L.ff);
                L.ff_silu = true;
                active_bytes += (uint64_t)3 * L.ff * W * 2;
            } else if (kind == "moe") {
                L.ff_kind = NVX_FF_ROUTED;
                L.route_kind = NVX_ROUTE_SIGMOID_BIAS;           // (no bias, one group: the scores alone pick and weigh)
                L.ff = (int)mlp["expert"]["ff"].as_int();
                L.n_expert = (int)mlp["router"]["experts"].as_int(); L.top = (int)mlp["router"]["top"].as_int();
                if (!cfg_positive(err, "mlp.expert.ff", L.ff) || !cfg_positive(err, "mlp.router.experts", L.n_expert, MOE_ROUTE_MAX_EXPERTS) || !cfg_positive(err, "mlp.router.top", L.top, L.n_expert)) return nullptr;
                std::vector<std::pair<std::string, int>> g, u, d;
                for (int e = 0; e < L.n_expert; e++) {
                    const std::string pe = pf + "e" + std::to_string(e) + ".";
                    g.push_back({pe + "gate", L.ff}); u.push_back({pe + "up", L.ff}); d.push_back({pe + "down", W});
                }
                L.e_gate = ld.rows(g, W); L.e_up = ld.rows(u, W); L.e_down = ld.rows(d, L.ff);
                L.ff_silu = true;
                L.weight_in = true;
                L.route = ld.rows({{pf + "router", L.n_expert}}, W);
                M.max_proj = std::max(M.max_proj, L.route.N);
                M.max_top = std::max(M.max_top, L.top);
                M.max_expert = std::max(M.max_expert, L.n_expert);
                active_bytes += ((uint64_t)L.n_expert * W + (uint64_t)L.top * 3 * L.ff * W) * 2;
            } else { err = at + "unknown mlp.kind '" + kind + "'"; return nullptr; }
            M.max_ff = std::max(M.max_ff, L.ff);
        }
    }
    if (!ld.err.empty()) { err = ld.err; return nullptr; }
    for (int il = 0; il < nl; il++) {
        const NvxLayer &L = M.layers[(size_t)il];
        NvxRun r; r.layer = il;
        r.plane = L.type == NVX_MLSTM ? M.n_state_runs++ : M.n_cache_runs++;
        if (L.type == NVX_GQ && L.conv_taps > 1) r.side_state = M.n_state_runs++;
        M.runs.push_back(r);
    }
    HParams &hp = m->hp;
    hp.arch = "vuzazen";
    hp.n_embd = W; hp.n_vocab = V; hp.n_vocab_local = V; hp.n_layer = nl; hp.n_layer_runs = nl;
    hp.n_head = M.layers[0].heads; hp.n_head_kv = M.layers[0].kv_heads; hp.head_dim = M.layers[0].dim; hp.eps = M.eps;
    hp.n_head_full = hp.n_head; hp.n_head_kv_full = hp.n_head_kv;
    hp.n_expert = M.max_expert; hp.n_expert_used = M.max_top;
    m->bytes_per_token = active_bytes;
    m->desc = "vuzazen " + std::to_string(nl) + " layers width " + std::to_string(W) + " BF16";
    status = 0;
    return m;
}

}  // namespace mi355
