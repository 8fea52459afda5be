// config_model.h — what the loaders of the folder models (config.json + model.safetensors, bf16 weights) share: reading the configuration, checking every
// tensor against it on the way to the device, and laying out the order of layer runs with its looped span.  One loader per design (novorax.cc, fidepel.cc,
// tuterax.cc, dinilorn.cc, vuzazen.cc, rarutar.cc); config_model_load picks it by the configuration's "architecture".
#pragma once

#include <algorithm>
#include <cmath>
#include <cstring>
#include <string>
#include <vector>

#include "json.h"
#include "runtime.h"
#include "safetensors.h"

namespace mi355 {

struct Bf16Loader {
    SafeTensorsFile st;
    Model *m = nullptr;
    std::string err;
    uint64_t bytes = 0;

    void *dev(const void *host, size_t n) {
        if (!err.empty()) return nullptr;
        void *p = nullptr;
        if (hipMalloc(&p, n ? n : 16) != hipSuccess) { err = "device allocation of " + std::to_string(n) + " bytes failed"; return nullptr; }
        m->arenas.push_back((uint8_t *)p);
        if (n && hipMemcpy(p, host, n, hipMemcpyHostToDevice) != hipSuccess) { err = "upload failed"; return nullptr; }
        bytes += n;
        return p;
    }
    const SafeTensor *need(const std::string &name, const char *dtype, std::initializer_list<int64_t> shape) {
        if (!err.empty()) return nullptr;
        const SafeTensor *t = st.find(name);
        if (!t) { err = "tensor '" + name + "' missing"; return nullptr; }
        if (t->dtype != dtype) { err = "tensor '" + name + "' is " + t->dtype + ", expected " + dtype; return nullptr; }
        if (t->shape.size() != shape.size() || !std::equal(shape.begin(), shape.end(), t->shape.begin())) {
            std::string want, have;
            for (int64_t d : shape) want += (want.empty() ? "" : ", ") + std::to_string(d);
            for (int64_t d : t->shape) have += (have.empty() ? "" : ", ") + std::to_string(d);
            err = "tensor '" + name + "' has shape [" + have + "], the configuration asks for [" + want + "]";
            return nullptr;
        }
        return t;
    }
    // several [rows_i][K] bf16 tensors under each other as one device matrix (an empty name: rows of zeros)
    BfMat rows(const std::vector<std::pair<std::string, int>> &parts, int K) {
        BfMat o;
        std::vector<unsigned short> host;
        for (const auto &pr : parts) {
            if (pr.first.empty()) { host.insert(host.end(), (size_t)pr.second * K, 0); o.N += pr.second; continue; }
            const SafeTensor *t = need(pr.first, "BF16", {pr.second, K});
            if (!t) return o;
            const unsigned short *s = (const unsigned short *)t->data;
            host.insert(host.end(), s, s + (size_t)pr.second * K);
            o.N += pr.second;
        }
        o.K = K;
        o.w = (unsigned short *)dev(host.data(), host.size() * 2);
        return o;
    }
    // several [N][K_i] bf16 tensors side by side as one device matrix
    BfMat cols(const std::vector<std::pair<std::string, int>> &parts, int N) {
        BfMat o;
        int K = 0, at = 0;
        for (const auto &pr : parts) K += pr.second;
        std::vector<unsigned short> host((size_t)N * K);
        for (const auto &pr : parts) {
            const SafeTensor *t = need(pr.first, "BF16", {N, pr.second});
            if (!t) return o;
            const unsigned short *s = (const unsigned short *)t->data;
            for (int n = 0; n < N; n++) std::copy(s + (size_t)n * pr.second, s + (size_t)(n + 1) * pr.second, host.begin() + (ptrdiff_t)((size_t)n * K + at));
            at += pr.second;
        }
        o.N = N; o.K = K;
        o.w = (unsigned short *)dev(host.data(), host.size() * 2);
        return o;
    }
    static float widen(unsigned short b) { const uint32_t u = (uint32_t)b << 16; float f; memcpy(&f, &u, 4); return f; }
    float *vec(const std::string &name, int n, float mult = 1.0f) {
        const SafeTensor *t = need(name, "BF16", {n});
        if (!t) return nullptr;
        std::vector<float> h((size_t)n);
        const unsigned short *s = (const unsigned short *)t->data;
        for (int i = 0; i < n; i++) h[(size_t)i] = widen(s[i]) * mult;
        return (float *)dev(h.data(), h.size() * 4);
    }
    // a layer norm's [n] weight and, behind it, its [n] bias (tensor name + ".b")
    float *norm_pair(const std::string &name, int n) {
        const SafeTensor *w = need(name, "BF16", {n}), *b = w ? need(name + ".b", "BF16", {n}) : nullptr;
        if (!b) return nullptr;
        std::vector<float> h((size_t)2 * n);
        for (int i = 0; i < n; i++) { h[(size_t)i] = widen(((const unsigned short *)w->data)[i]); h[(size_t)(n + i)] = widen(((const unsigned short *)b->data)[i]); }
        return (float *)dev(h.data(), h.size() * 4);
    }
    // w reads rows behind this layer norm (norm_pair of w.K entries): its rows' sums with the norm's weight and bias, made on the device in f32
    void reads_layer_norm(BfMat &w, const float *norm) {
        if (!err.empty() || !w.w || !norm) return;
        void *p = nullptr;
        if (hipMalloc(&p, (size_t)2 * w.N * 4) != hipSuccess) { err = "device allocation of a norm's row sums failed"; return; }
        m->arenas.push_back((uint8_t *)p);
        w.ln = (float *)p;
        MMBArgs a;
        a.x = norm; a.ldx = w.K; a.w = w.w; a.ldw = w.K; a.y = w.ln; a.ldy = w.N; a.T = 2; a.N = w.N; a.K = w.K; a.f32 = 1;
        if (launch_mmb(a, nullptr) != hipSuccess) err = "a norm's row sums failed";
    }
    // several [rows_i][K] bf16 tensors under each other, widened to f32 and transposed: [K][sum of rows]
    float *rows_f32_transposed(const std::vector<std::pair<std::string, int>> &parts, int K) {
        size_t N = 0, at = 0;
        for (const auto &pr : parts) N += (size_t)pr.second;
        std::vector<float> h(N * (size_t)K);
        for (const auto &pr : parts) {
            const SafeTensor *t = need(pr.first, "BF16", {pr.second, K});
            if (!t) return nullptr;
            const unsigned short *s = (const unsigned short *)t->data;
            for (int r = 0; r < pr.second; r++, at++)
                for (int k = 0; k < K; k++) h[(size_t)k * N + at] = widen(s[(size_t)r * K + k]);
        }
        return (float *)dev(h.data(), h.size() * 4);
    }
    // radians per position of pair i of `dims` turning entries: base^(-2i / dims), made in double.  With a scaling object {factor, original, fast, slow} (YaRN):
    // blended towards 1 / factor of itself where the pair turns too slowly for the original context (ramp 0 below `lo`, 1 above `hi`); *mscale = the factor of cos and
    // sin, 0.1 ln(factor) + 1 then, else 1
    float *rot_table(double base, int dims, const Json &scaling, float *mscale) {
        std::vector<float> fr((size_t)std::max(dims / 2, 1), 0.0f);
        double factor = 1.0, lo = 0.0, hi = 0.0;
        const bool yarn = scaling.is_object() && dims > 0;
        if (mscale) *mscale = 1.0f;
        if (yarn) {
            factor = scaling["factor"].as_double(1.0);
            const double orig = scaling["original"].as_double(1.0), fast = scaling["fast"].as_double(32.0), slow = scaling["slow"].as_double(1.0);
            if (!(factor > 0.0) || !(orig > 0.0) || !(fast > 0.0) || !(slow > 0.0) || !(base > 1.0)) { if (err.empty()) err = "configuration: rot.scaling values must be positive"; return nullptr; }
            const auto corr = [&](double turns) { return dims * std::log(orig / (2.0 * M_PI * turns)) / (2.0 * std::log(base)); };
            lo = std::max(std::floor(corr(fast)), 0.0);
            hi = std::min(std::ceil(corr(slow)), (double)(dims - 1));
            if (mscale) *mscale = (float)(0.1 * std::log(factor) + 1.0);
        }
        for (int i = 0; i < dims / 2; i++) {
            double f = std::pow(base, -2.0 * i / dims);
            if (yarn) {
                const double ramp = std::min(1.0, std::max(0.0, (i - lo) / std::max(hi - lo, 0.001)));
                f = f / factor * ramp + f * (1.0 - ramp);
            }
            fr[(size_t)i] = (float)f;
        }
        return (float *)dev(fr.data(), fr.size() * 4);
    }
    // rows of a [rows][K] tensor whose row count the configuration does not name (a low-rank projection's inner size): -1 (err set) if absent or not 2-d
    int rows_of(const std::string &name, int K) {
        if (!err.empty()) return -1;
        const SafeTensor *t = st.find(name);
        if (!t) { err = "tensor '" + name + "' missing"; return -1; }
        if (t->shape.size() != 2 || t->shape[1] != K || t->shape[0] < 1 || t->shape[0] > (1 << 24)) { err = "tensor '" + name + "' must be [rows][" + std::to_string(K) + "]"; return -1; }
        return (int)t->shape[0];
    }
    // several [rows_i][K] bf16 tensors under each other, widened to f32 (small per-channel tables a kernel reads as floats)
    float *rows_f32(const std::vector<std::pair<std::string, int>> &parts, int K) {
        std::vector<float> host;
        for (const auto &pr : parts) {
            const SafeTensor *t = need(pr.first, "BF16", {pr.second, K});
            if (!t) return nullptr;
            const unsigned short *s = (const unsigned short *)t->data;
            for (size_t i = 0; i < (size_t)pr.second * K; i++) host.push_back(widen(s[i]));
        }
        return (float *)dev(host.data(), host.size() * 4);
    }
    // a tensor that holds ONE number, as n copies of it: a norm weight shared by all coordinates takes the kernels' per-coordinate form
    float *scalar_as_vec(const std::string &name, int n) {
        const SafeTensor *t = need(name, "BF16", {});
        if (!t) return nullptr;
        std::vector<float> h((size_t)n, widen(*(const unsigned short *)t->data));
        return (float *)dev(h.data(), h.size() * 4);
    }
    // a [heads * D][R] bf16 tensor transposed inside every head: [heads][R][D] (a per-head product with the transpose)
    BfMat head_transposed(const std::string &name, int heads, int D, int R) {
        BfMat o;
        const SafeTensor *t = need(name, "BF16", {(int64_t)heads * D, R});
        if (!t) return o;
        const unsigned short *s = (const unsigned short *)t->data;
        std::vector<unsigned short> tr((size_t)heads * R * D);
        for (int h = 0; h < heads; h++)
            for (int d = 0; d < D; d++)
                for (int r = 0; r < R; r++) tr[((size_t)h * R + r) * D + d] = s[((size_t)h * D + d) * R + r];
        o.w = (unsigned short *)dev(tr.data(), tr.size() * 2);
        o.N = R; o.K = D;
        return o;
    }
    // the embedding table with the row stride launch_get_rows expects
    BfMat embedding(const std::string &name, int V, int W) {
        BfMat o;
        const SafeTensor *t = need(name, "BF16", {V, W});
        if (!t) return o;
        const size_t rb = dev_row_bytes(T_BF16, W);
        std::vector<uint8_t> host((size_t)V * rb, 0);
        for (int r = 0; r < V; r++) memcpy(host.data() + (size_t)r * rb, t->data + (size_t)r * W * 2, (size_t)W * 2);
        o.w = (unsigned short *)dev(host.data(), host.size());
        o.N = V; o.K = W;
        return o;
    }
};

inline bool cfg_positive(std::string &err, const char *what, int64_t v, int64_t hi = 1 << 24) {
    if (v >= 1 && v <= hi) return true;
    err = std::string("configuration: ") + what + " = " + std::to_string(v) + " is out of range";
    return false;
}

// The order of layer runs from the configuration's "loop" {start, stop, times}: layers before the span once, the span `times` times with the same weights,
// the rest once.  on_run(layer, pass): pass >= 0 for the first layer of pass `pass` of the span, -1 elsewhere.  false (err set) for a span out of range.
template <class F>
bool cfg_layer_runs(const Json &loop, int n_layer, std::string &err, int &times_out, F on_run) {
    int a = 0, b = 0, times = 0;
    if (loop.is_object()) {
        a = (int)loop["start"].as_int(0); b = (int)loop["stop"].as_int(0); times = (int)loop["times"].as_int(1);
        if (a < 0 || b > n_layer || times < 0 || times > 4096) { err = "configuration: loop start / stop / times out of range"; return false; }
        if (b <= a || times < 1) { a = b = 0; times = 0; }
    }
    for (int i = 0; i < a; i++) on_run(i, -1);
    for (int t = 0; t < times; t++) for (int i = a; i < b; i++) on_run(i, i == a ? t : -1);
    for (int i = b; i < n_layer; i++) on_run(i, -1);
    times_out = times;
    return true;
}

// from this many (token, rank) pairs on a routed feed-forward groups the pairs by expert and runs every expert's rows as one batch (fidepel.cc)
bool nvx_routed_as_groups(const NvxLayer &L, int T);

// the designs' loaders: cfg is the parsed config.json of `dir`, ld has model.safetensors open and ld.m set
Model *novorax_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status);
Model *fidepel_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status);
Model *tuterax_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status);
Model *dinilorn_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status);
Model *vuzazen_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status);
Model *rarutar_build(const Json &cfg, const std::string &dir, Bf16Loader &ld, std::string &err, int &status);

}  // namespace mi355
