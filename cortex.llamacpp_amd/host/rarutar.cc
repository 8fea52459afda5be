// rarutar.cc — loading a Rarutar folder, its recurrences and its side-by-side mixers inside Context (novorax.h describes the design, config_model.h the shared
// loader).
//
// A layer is x += mixer(norm(x)), then x += ff(norm(x)) with layer norms in front of the sublayers only: a norm vector holds weights and biases one behind the other,
// every matrix that reads normed rows knows its rows' sums with both (Bf16Loader::reads_layer_norm), so that a step of few rows norms inside its products
// (nvx_linear) and no launch stands between two sublayers (nvx_close_linear).  Attention of either kind is the grouped-query attention of fidepel.cc with further
// switches.  Two mixers side by side read ONE projection [left q ; k ; v ; g | right q ; k ; v ; g ; a1], write their outputs side by side into one row - each times its
// constant, which the attention applies behind its gate and the recurrence carries in its norm's weight - and close with ONE product against their W_o side by side.
// Gated linear attention and the state-space recurrence are two uses of gated_scan.hip.
#include "config_model.h"

namespace mi355 {

void set_error(const char *fmt, ...);

#define RRT_TRY(expr)                                                                              \
    do {                                                                                           \
        hipError_t e_ = (expr);                                                                    \
        if (e_ != hipSuccess) {                                                                    \
            set_error("%s failed: %s (%s:%d)", #expr, hipGetErrorString(e_), __FILE__, __LINE__);  \
            return e_;                                                                             \
        }                                                                                          \
    } while (0)

namespace {

struct Reader {
    Bf16Loader &ld;
    NovoraxModel &M;
    std::string &err;
    std::string at;                                             // "configuration: layer i: "
    int W;

    bool heads_of(const Json &mx, NvxLayer &L) {
        L.heads = (int)mx["heads"].as_int(); L.kv_heads = (int)mx["kv_heads"].as_int(L.heads); L.dim = (int)mx["dim"].as_int(); L.vdim = (int)mx["vdim"].as_int(L.dim);
        if (!cfg_positive(err, "mixer.heads", L.heads, 4096) || !cfg_positive(err, "mixer.kv_heads", L.kv_heads, L.heads) || !cfg_positive(err, "mixer.dim", L.dim, 1 << 16) ||
            !cfg_positive(err, "mixer.vdim", L.vdim, 1 << 16)) return false;
        if (L.heads % L.kv_heads != 0) { err = at + "mixer.heads must be a multiple of mixer.kv_heads"; return false; }
        return true;
    }
    bool attention_of(const Json &mx, NvxLayer &L) {            // what both attentions share: heads, scale, rotation, mask size
        L.type = NVX_GQ;
        if (!heads_of(mx, L)) return false;
        if (!gq_attn_shape_ok(L.heads, L.kv_heads, L.dim, L.vdim)) {
            err = "attention: dim " + std::to_string(L.dim) + " / vdim " + std::to_string(L.vdim) + " is beyond what the attention kernel holds per lane (512)";
            return false;
        }
        L.scale = (float)mx["scale"].as_double(1.0);
        const Json &rot = mx["rot"];
        L.rot_dims = rot.is_object() ? (int)rot["dims"].as_int(0) : 0;
        if (L.rot_dims > L.dim || (L.rot_dims & 1) || L.rot_dims < 0) { err = at + "rot.dims must be even and at most mixer.dim"; return false; }
        if (L.rot_dims > 0) {
            const double base = rot["base"].as_double(10000.0);
            if (!(base > 0.0)) { err = at + "rot.base must be positive"; return false; }
            L.rot_freq = ld.rot_table(base, L.rot_dims, rot["scaling"], &L.rot_mscale);
        }
        M.max_q = std::max(M.max_q, L.heads * L.dim);
        return true;
    }
    bool mask_of(const Json &mx, int &size) {                   // 0: every earlier position
        size = 0;
        if (!mx["mask"].is_object()) return true;
        size = (int)mx["mask"]["size"].as_int(0);
        if (!cfg_positive(err, "mixer.mask.size", size, 1 << 30)) return false;
        M.max_window = std::max(M.max_window, size);
        return true;
    }
};

int padded(int n) { return (n + 3) & ~3; }                      // (columns that start on 16-byte boundaries)

}  // namespace

Model *rarutar_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status) {
    (void)dir;
    status = -102;
    Model *const m = ld.m;
    NovoraxModel &M = *m->nvx;
    M.design = "rarutar";
    M.norm_off = 0.0f;
    M.layer_norm = true;
    const int W = (int)cfg["width"].as_int(), V = (int)cfg["vocab"].as_int();
    if (!cfg_positive(err, "width", W) || !cfg_positive(err, "vocab", V)) return nullptr;
    M.width = W; M.n_vocab = V;
    M.eps = (float)cfg["norm"]["eps"].as_double(1e-5);
    M.embed_scale = (float)cfg["embedding"]["scale"].as_double(1.0);
    const Json &layers = cfg["layers"];
    if (!layers.is_array() || layers.size() == 0 || layers.size() > 1024) { err = "configuration: 'layers' must list 1 .. 1024 layers"; return nullptr; }
    const int nl = (int)layers.size();

    M.embed = ld.embedding("embed", V, W);                      // the table the tokens' rows come from ...
    M.head = ld.rows({{"embed", V}}, W);                        // ... is the output head too (dense rows for the linear kernels)
    M.final_norm = ld.norm_pair("final.norm", W);
    ld.reads_layer_norm(M.head, M.final_norm);
    uint64_t active_bytes = ((uint64_t)V * W + W) * 2;          // what one token reads of the weights: the head and a table row, then every layer's matrices

    M.layers.resize((size_t)nl);
    for (int il = 0; il < nl && ld.err.empty(); il++) {
        const Json &lc = layers.at((size_t)il), &mx = lc["mixer"];
        NvxLayer &L = M.layers[(size_t)il];
        const std::string p = "l" + std::to_string(il) + ".", pm = p + "mix.", type = lc["type"].as_string();
        Reader rd{ld, M, err, "configuration: layer " + std::to_string(il) + ": ", W};
        L.norm1 = ld.norm_pair(p + "norm1", W);
        if (type == "parallel") {
            L.type = NVX_BESIDE;
            L.mixers.resize(2);
            NvxLayer &A = L.mixers[0], &B = L.mixers[1];
            const Json &ml = mx["left"], &mr = mx["right"];
            if (!rd.attention_of(ml, A) || !rd.mask_of(ml, A.window)) return nullptr;
            A.out_mult = (float)mx["left_scale"].as_double(1.0);
            const int NQ = A.heads * A.dim, NK = A.kv_heads * A.dim, NV = A.kv_heads * A.vdim;
            A.off_gate = NQ + NK + NV;
            const int left = A.off_gate + A.heads;
            B.type = NVX_GLA;
            if (!rd.heads_of(mr, B)) return nullptr;
            B.kv_heads = B.heads;
            if (!gated_scan_shape_ok(B.heads, 1, B.dim, B.vdim)) { err = "gated linear attention: dim " + std::to_string(B.dim) + " is beyond what the recurrence kernel stages (" + std::to_string(GATED_SCAN_MAX_DIM) + ")"; return nullptr; }
            const double tau = mr["tau"].as_double(1.0);
            if (!(tau > 0.0)) { err = rd.at + "mixer.right.tau must be positive"; return nullptr; }
            B.inv_tau = (float)(1.0 / tau);
            B.scale = (float)(1.0 / std::sqrt((double)B.dim));
            const int RQ = B.heads * B.dim, RV = B.heads * B.vdim;
            B.rank_a = ld.rows_of(pm + "right.a1", W);
            if (B.rank_a < 0) break;
            B.off_p = padded(left);
            B.off_g = 2 * RQ + RV;
            B.off_a = padded(B.off_g + RV);
            B.off_att = A.heads * A.vdim;
            const int all = B.off_p + B.off_a + B.rank_a;
            L.proj = ld.rows({{pm + "left.q", NQ}, {pm + "left.k", NK}, {pm + "left.v", NV}, {pm + "left.g", A.heads}, {"", B.off_p - left},
                              {pm + "right.q", RQ}, {pm + "right.k", RQ}, {pm + "right.v", RV}, {pm + "right.g", RV}, {"", B.off_a - B.off_g - RV}, {pm + "right.a1", B.rank_a},
                              {"", padded(all) - all}}, W);
            ld.reads_layer_norm(L.proj, L.norm1);
            B.a2 = ld.rows({{pm + "right.a2", RQ}}, B.rank_a);
            B.a2_bias = ld.vec(pm + "right.a2.b", RQ);
            B.mix_norm = ld.vec(pm + "right.norm", B.vdim, (float)mx["right_scale"].as_double(1.0));   // (the constant rides in the norm's weight)
            L.o = ld.cols({{pm + "left.o", B.off_att}, {pm + "right.o", RV}}, W);
            L.heads = A.heads; L.kv_heads = A.kv_heads; L.dim = A.dim; L.vdim = A.vdim;
            M.max_qa = std::max(M.max_qa, RQ);
            M.max_att = std::max(M.max_att, B.off_att + RV);
            active_bytes += ((uint64_t)L.proj.N * W + (uint64_t)RQ * B.rank_a + (uint64_t)W * L.o.K) * 2;
        } else if (type == "attention") {
            if (!rd.attention_of(mx, L) || !rd.mask_of(mx, L.chunk)) return nullptr;
            if (L.vdim != L.dim) { err = rd.at + "mixer.vdim must equal mixer.dim (the values are the keys)"; return nullptr; }
            L.v_is_k = true;
            L.qk_unit = true;
            const int NQ = L.heads * L.dim, NK = L.kv_heads * L.dim, all = NQ + NK + L.heads;
            L.off_gate = NQ + NK;
            L.proj = ld.rows({{pm + "q", NQ}, {pm + "k", NK}, {pm + "g", L.heads}, {"", padded(all) - all}}, W);
            ld.reads_layer_norm(L.proj, L.norm1);
            L.sink = ld.vec(pm + "sink", L.heads);
            L.o = ld.rows({{pm + "o", W}}, L.heads * L.vdim);
            M.max_att = std::max(M.max_att, L.heads * L.vdim);
            active_bytes += ((uint64_t)L.proj.N * W + (uint64_t)W * L.o.K) * 2;
        } else if (type == "mamba2") {
            L.type = NVX_SSD;
            L.heads = (int)mx["heads"].as_int(); L.vdim = (int)mx["vdim"].as_int(); L.dim = (int)mx["state"].as_int(); L.kv_heads = (int)mx["groups"].as_int(1);
            L.conv_taps = (int)mx["conv"].as_int(1); L.norm_parts = (int)mx["norm_groups"].as_int(1);
            if (!cfg_positive(err, "mixer.heads", L.heads, 4096) || !cfg_positive(err, "mixer.vdim", L.vdim, 1 << 16) || !cfg_positive(err, "mixer.state", L.dim, GATED_SCAN_MAX_DIM) ||
                !cfg_positive(err, "mixer.groups", L.kv_heads, L.heads) || !cfg_positive(err, "mixer.conv", L.conv_taps, 64) || !cfg_positive(err, "mixer.norm_groups", L.norm_parts, L.heads * L.vdim)) return nullptr;
            const int H = L.heads, inner = H * L.vdim, GN = L.kv_heads * L.dim;
            if (H % L.kv_heads != 0) { err = rd.at + "mixer.heads must be a multiple of mixer.groups"; return nullptr; }
            if (inner % L.norm_parts != 0) { err = rd.at + "mixer.norm_groups must divide heads * vdim"; return nullptr; }
            const int all = 2 * inner + 2 * GN + H;
            L.off_a = 2 * inner + 2 * GN;
            L.proj = ld.rows({{pm + "in", all}}, W);
            ld.reads_layer_norm(L.proj, L.norm1);
            L.conv_wt = ld.rows_f32_transposed({{pm + "conv", L.conv_channels()}}, L.conv_taps);
            L.conv_b = ld.vec(pm + "conv.b", L.conv_channels());
            L.dt_bias = ld.vec(pm + "dt_bias", H);
            L.A_log = ld.vec(pm + "A_log", H);
            L.skip = ld.vec(pm + "D", H);
            L.mix_norm = ld.vec(pm + "norm", inner);
            L.o = ld.rows({{pm + "o", W}}, inner);
            M.max_q = std::max(M.max_q, padded(L.conv_channels()));
            M.max_att = std::max(M.max_att, inner);
            active_bytes += ((uint64_t)L.proj.N * W + (uint64_t)W * inner) * 2;
        } else { err = rd.at + "unknown type '" + type + "'"; return nullptr; }
        M.max_proj = std::max(M.max_proj, padded(L.proj.N));
        const Json &mlp = lc["mlp"];
        if (mlp.is_object()) {
            const std::string pf = p + "mlp.", kind = mlp["kind"].as_string();
            if (kind != "dense") { err = rd.at + "unknown mlp.kind '" + kind + "'"; return nullptr; }
            L.norm2 = ld.norm_pair(p + "norm2", W);
            L.ff_kind = NVX_FF_DENSE;
            L.ff = (int)mlp["ff"].as_int();
            L.ff_limit = (float)mlp["limit"].as_double(0.0);
            if (!cfg_positive(err, "mlp.ff", L.ff)) return nullptr;
            if (!(L.ff_limit > 0.0f)) { err = rd.at + "mlp.limit must be positive"; return nullptr; }
            L.gate = ld.rows({{pf + "gate", L.ff}}, W);
            L.up = ld.rows({{pf + "up", L.ff}}, W);
            ld.reads_layer_norm(L.gate, L.norm2);
            ld.reads_layer_norm(L.up, L.norm2);
            L.down_ff = ld.rows({{pf + "down", W}}, L.ff);
            M.max_ff = std::max(M.max_ff, L.ff);
            active_bytes += (uint64_t)3 * L.ff * W * 2;
        }
    }
    if (err.empty()) err = ld.err;
    if (!err.empty()) return nullptr;
    for (int il = 0; il < nl; il++) {
        const NvxLayer &L = M.layers[(size_t)il];
        NvxRun r; r.layer = il;
        r.plane = L.type == NVX_SSD ? M.n_state_runs++ : M.n_cache_runs++;
        if (L.type == NVX_BESIDE) r.side_state = M.n_state_runs++;
        M.runs.push_back(r);
    }
    HParams &hp = m->hp;
    hp.arch = "rarutar";
    hp.n_embd = W; hp.n_vocab = V; hp.n_vocab_local = V; hp.n_layer = nl; hp.n_layer_runs = nl;
    hp.n_head = M.layers[0].heads; hp.n_head_kv = M.layers[0].kv_heads; hp.head_dim = M.layers[0].dim; hp.eps = M.eps;
    hp.n_head_full = hp.n_head; hp.n_head_kv_full = hp.n_head_kv;
    m->bytes_per_token = active_bytes;
    m->desc = "rarutar " + std::to_string(nl) + " layers width " + std::to_string(W) + " BF16";
    status = 0;
    return m;
}

// ------------------------------------------------------------------------------------------ mixers
hipError_t Context::nvx_beside_mixers(const NvxLayer &L, const NvxRun &r, int T) {
    const int LD_P = L.proj.N, LD_O = L.o.K;
    RRT_TRY(nvx_linear(L.proj, x_, model->nvx->width, T, nvx_a_, LD_P, MMB_STORE, nullptr, 1.0f, L.norm1));
    for (const NvxLayer &X : L.mixers) {
        if (X.type == NVX_GQ) RRT_TRY(nvx_gq_heads(X, r, T, nvx_a_ + X.off_p, LD_P, nvx_att_ + X.off_att, LD_O));
        else if (X.type == NVX_GLA) RRT_TRY(nvx_gla_heads(X, r.side_state, T, nvx_a_ + X.off_p, LD_P, nvx_att_ + X.off_att, LD_O));
        else return hipErrorInvalidValue;
    }
    RRT_TRY(nvx_close_linear(L.o, nvx_att_, LD_O, T, L.norm1b));
    prof_mark("side_by_side");
    return hipSuccess;
}

hipError_t Context::nvx_gla_mixer(const NvxLayer &L, const NvxRun &r, int T) {
    const int LD_P = L.proj.N, LD_O = L.heads * L.vdim;
    RRT_TRY(nvx_linear(L.proj, x_, model->nvx->width, T, nvx_a_, LD_P, MMB_STORE, nullptr, 1.0f, L.norm1));
    RRT_TRY(nvx_gla_heads(L, r.plane, T, nvx_a_, LD_P, nvx_att_, LD_O));
    RRT_TRY(nvx_close_linear(L.o, nvx_att_, LD_O, T, L.norm1b));
    prof_mark("gated_linear_attention");
    return hipSuccess;
}

// the heads' normed and gated outputs -> out[t][heads * vdim] from the projection rows p
hipError_t Context::nvx_gla_heads(const NvxLayer &L, int state_set, int T, const float *p, int LD_P, float *out, int ld_out) {
    const NovoraxModel &M = *model->nvx;
    const int H = L.heads, D = L.dim, VD = L.vdim;
    const size_t TU = cp.n_ubatch;
    bool batch = false;                                         // some segment holds several rows: its decays are made for all rows at once
    for (const auto &wv : nvx_waves_) for (int s = 0; s < wv.second; s++) batch = batch || h_seg_[TU + (size_t)(wv.first + s)] > 1;
    if (batch) RRT_TRY(launch_gated_decay(p + L.off_a, LD_P, T, L.rank_a, L.a2.w, L.a2_bias, L.inv_tau, H * D, nvx_qa_, H * D, stream_));
    GatedScanArgs ga{};
    ga.p = p; ga.ld_p = LD_P; ga.off_q = 0; ga.off_k = H * D; ga.off_v = 2 * H * D; ga.share = 1; ga.q_scale = L.scale;
    ga.alpha = nvx_qa_; ga.ld_alpha = H * D; ga.lr_bias = L.a2_bias; ga.rank = L.rank_a; ga.off_lr = L.off_a; ga.inv_tau = L.inv_tau;
    ga.S = nvx_S_[(size_t)state_set]; ga.o = nvx_o_; ga.ld_o = H * VD; ga.H = H; ga.D = D; ga.VD = VD;
    ga.ld_y = ld_out; ga.gate = p + L.off_g; ga.ld_gate = LD_P; ga.norm_w = L.mix_norm; ga.eps = M.eps;
    ga.w_A = nvx_gs_A_; ga.w_q = nvx_gs_q_; ga.w_k = nvx_gs_q_ + TU * (size_t)(H * D); ga.w_g = nvx_gs_g_; ga.w_S = nvx_gs_S_;
    for (const auto &wv : nvx_waves_) {
        const int *start = h_seg_ + wv.first, *len = h_seg_ + TU + wv.first;
        const int rows = start[wv.second - 1] + len[wv.second - 1] - start[0];
        ga.seg_start = d_seg_ + wv.first; ga.seg_len = d_seg_ + TU + wv.first; ga.seg_slot = d_seg_ + 2 * TU + wv.first; ga.n_seg = wv.second;
        ga.row0 = start[0]; ga.max_len = *std::max_element(len, len + wv.second);
        ga.lr_w = ga.max_len == 1 ? L.a2.w : nullptr;
        const bool closes = ga.max_len == 1 && gated_step_closes(VD);
        ga.y = closes ? out : nullptr;
        RRT_TRY(launch_gated_scan(ga, stream_));
        const size_t r0 = (size_t)start[0];
        if (!closes)
            RRT_TRY(launch_mlstm_out(nvx_o_ + r0 * (size_t)(H * VD), H * VD, p + r0 * (size_t)LD_P, LD_P, L.off_g, L.mix_norm, rows, H, VD, M.eps, out + r0 * (size_t)ld_out, ld_out,
                                     stream_, 0, MLSTM_GATE_SILU));
    }
    return hipSuccess;
}

hipError_t Context::nvx_ssd_mixer(const NvxLayer &L, const NvxRun &r, int T) {
    const NovoraxModel &M = *model->nvx;
    const int H = L.heads, D = L.dim, VD = L.vdim, G = L.kv_heads, inner = H * VD, C = L.conv_channels(), LD_P = padded(L.proj.N), LD_C = padded(C);
    const size_t TU = cp.n_ubatch;
    RRT_TRY(nvx_linear(L.proj, x_, M.width, T, nvx_a_, LD_P, MMB_STORE, nullptr, 1.0f, L.norm1));
    float *const xbc = nvx_a_ + inner, *const conv_state = nvx_n_[(size_t)r.plane];
    GatedScanArgs ga{};
    ga.off_v = 0; ga.off_k = inner; ga.off_q = inner + G * D; ga.share = H / G; ga.q_scale = 1.0f;
    ga.dt = nvx_a_ + L.off_a; ga.ld_dt = LD_P; ga.dt_bias = L.dt_bias; ga.A_log = L.A_log; ga.skip = L.skip;
    ga.S = nvx_S_[(size_t)r.plane]; ga.o = nvx_o_; ga.ld_o = inner; ga.H = H; ga.D = D; ga.VD = VD;
    ga.w_A = nvx_gs_A_; ga.w_p = nvx_gs_p_; ga.w_s = nvx_gs_p_ + TU * (size_t)H; ga.w_g = nvx_gs_g_; ga.w_S = nvx_gs_S_;
    for (const auto &wv : nvx_waves_) {
        const int *start = h_seg_ + wv.first, *len = h_seg_ + TU + wv.first;
        const int rows = start[wv.second - 1] + len[wv.second - 1] - start[0];
        const size_t r0 = (size_t)start[0];
        ga.seg_start = d_seg_ + wv.first; ga.seg_len = d_seg_ + TU + wv.first; ga.seg_slot = d_seg_ + 2 * TU + wv.first; ga.n_seg = wv.second;
        ga.row0 = start[0]; ga.max_len = *std::max_element(len, len + wv.second);
        const bool step = ga.max_len == 1;
        ConvMove mv{};
        if (step) {                                             // the convolution is part of the step; the launch behind it moves its state on
            ga.p = xbc; ga.ld_p = LD_P;
            ga.conv_wt = L.conv_wt; ga.conv_b = L.conv_b; ga.conv_state = conv_state; ga.conv_taps = L.conv_taps; ga.conv_C = C;
            if (L.conv_taps > 1) mv = ConvMove{conv_state, xbc + r0 * (size_t)LD_P, LD_P, C, L.conv_taps, ga.seg_slot};
        } else {
            RRT_TRY(launch_conv_silu(xbc + r0 * (size_t)LD_P, LD_P, C, L.conv_wt, L.conv_b, L.conv_taps, conv_state, d_seg_ + 5 * TU + r0, d_seq_ + r0, rows, nvx_q_ + r0 * (size_t)LD_C, LD_C, stream_));
            RRT_TRY(launch_conv_state(xbc, LD_P, C, L.conv_taps, conv_state, ga.seg_start, ga.seg_len, ga.seg_slot, ga.n_seg, stream_));
            ga.p = nvx_q_; ga.ld_p = LD_C;
            ga.conv_wt = nullptr; ga.conv_b = ga.conv_state = nullptr;
        }
        RRT_TRY(launch_gated_scan(ga, stream_));
        RRT_TRY(launch_gated_norm(nvx_o_ + r0 * (size_t)inner, inner, nvx_a_ + r0 * (size_t)LD_P, LD_P, L.mix_norm, rows, L.norm_parts, inner / L.norm_parts, M.eps,
                                  nvx_att_ + r0 * (size_t)inner, inner, mv, stream_));
    }
    RRT_TRY(nvx_close_linear(L.o, nvx_att_, inner, T, L.norm1b));
    prof_mark("state_space");
    return hipSuccess;
}

}  // namespace mi355
