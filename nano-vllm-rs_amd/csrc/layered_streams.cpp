// layered_streams.cpp — the streams layout of layer-list models (layered_model.h): the residual is a set of parallel streams.  Sublayer: u = sum_s in_s x_s, y = f(layer norm(u)),
// x_q <- sum_s mix_sq x_s + out_q y.  Mixers: softmax attention with projection biases, a rotation of number pairs with stretched frequencies, unit norms behind it, values mixed
// with the first such layer's, an output gate.  Feed-forwards: gated GELU, or experts some of which return their input.  A sublayer's write and the next one's read and norm are
// one launch; the last write, the sum over the streams and the final norm happen on the rows whose logits are asked for.
#include <algorithm>
#include <cmath>
#include <cstring>
#include "layered_model.h"
#include "model_runner.h"
#include "kernels/kernels.h"

#define RC(expr) do { int _rc = (expr); if (_rc) return _rc; } while (0)

namespace nvr {

namespace {
inline int64_t pad16(int64_t n) { return (n + 15) / 16 * 16; }

template <class V, class T> void add_once(V &v, T x) { if (std::find(v.begin(), v.end(), x) == v.end()) v.push_back(x); }
template <class V, class T> size_t index_of(const V &v, T x) { return (size_t)(std::find(v.begin(), v.end(), x) - v.begin()); }
}

int LayeredModel::init_streams(nvr_model_runner &r) {
    const int64_t W = spec.width, V = spec.vocab, S = spec.streams, MT = r.max_tokens;
    auto named = [&](void **p, size_t bytes) {              // (the buffers the destructor frees by name)
        NVR_HIP_CHECK(hipMalloc(p, bytes ? bytes : 16));
        NVR_HIP_CHECK(hipMemset(*p, 0, bytes ? bytes : 16));
        return (int)NVR_OK;
    };
    lw.resize(spec.layers.size());
    int64_t max_nmix = 0, max_hv = 0, max_ff = 0, max_gv = 0, max_top = 0, max_f = 0, max_e2f = 0, max_ef = 0, max_experts = 0, max_router = 0, max_pairs = 0;
    for (size_t i = 0; i < spec.layers.size(); ++i) {
        const LayeredSpec::Layer &L = spec.layers[i]; LayerW &w = lw[i];
        if (L.mixer != LayeredSpec::ATTN_UNIT) return fail(NVR_ERR_UNSUPPORTED, "layer %zu: this mixer does not belong to the streams layout", i);
        const int64_t hd = L.heads * L.dim, kn = L.kv_heads * L.dim, vn = L.kv_heads * L.vdim, hv = L.heads * L.vdim, g = L.heads / L.kv_heads;
        for (int q = 0; q < (L.has_mlp ? 2 : 1); ++q) {
            RC(own(q ? &w.n2 : &w.n1, (size_t)W * 4));
            RC(own(&w.hin[q], (size_t)S * 4)); RC(own(&w.hout[q], (size_t)S * 4)); RC(own(&w.hmix[q], (size_t)(S * S) * 4));
        }
        w.qcol = 0; w.kcol = pad16(hd); w.vcol = w.kcol + pad16(kn); w.gcol = w.vcol + pad16(vn); w.nmix = w.gcol + pad16(hv);
        RC(named(&w.mix, (size_t)(w.nmix * W * esz))); RC(own(&w.wo, (size_t)(W * hv * esz)));
        RC(own(&w.bq, (size_t)hd * 4)); RC(own(&w.bk, (size_t)kn * 4)); RC(own(&w.bv, (size_t)vn * 4)); RC(own(&w.vmix, 4));
        const std::vector<float> f = rotation_frequencies(L);
        RC(own(&w.rfreq, f.size() * 4)); NVR_HIP_CHECK(hipMemcpy(w.rfreq, f.data(), f.size() * 4, hipMemcpyHostToDevice));
        add_once(attn_groups, g);
        // plain causal softmax: equal key and value sizes of 64 / 128 take the dense graph's kernels, prompts and portions its flash kernel, decoded tokens its split decode attention
        w.flash = bf16 && L.dim == L.vdim && nvr::kb::flash_prefill_ok((int)L.dim, (int)L.heads, (int)L.kv_heads);
        if (w.flash) {
            flash_kind(nvr::kb::flash_tile_positions((int)L.heads, (int)L.kv_heads));
            dec_ws_bytes = std::max(dec_ws_bytes, nvr::kb::attn_workspace_bytes(r.max_seqs, L.heads, L.dim, (r.max_pos + 255) / 256 * 256));
            max_pairs = std::max(max_pairs, r.max_seqs * L.kv_heads);
        }
        if (L.ff_kind == LayeredSpec::FF_GEGLU) {
            RC(own(&w.up, (size_t)(2 * L.ff * W * esz))); RC(own(&w.down, (size_t)(W * L.ff * esz)));      // up: gate rows, then up rows
            max_ff = std::max(max_ff, L.ff);
        } else if (L.ff_kind == LayeredSpec::FF_MOE_IDENT) {
            const int64_t fe = L.expert_ff, ne = L.experts + L.identity;
            RC(own(&w.router_op, (size_t)(pad16(ne) * W * esz))); RC(own(&w.ecorr, (size_t)ne * 4));
            RC(own(&w.egu, (size_t)(L.experts * 2 * fe * W * esz))); RC(own(&w.edown, (size_t)(L.experts * W * fe * esz)));
            max_top = std::max(max_top, L.top); max_e2f = std::max(max_e2f, L.top * 2 * fe); max_ef = std::max(max_ef, L.top * fe);
            max_experts = std::max(max_experts, L.experts); max_router = std::max(max_router, ne); max_f = std::max(max_f, fe);
        } else if (L.has_mlp) return fail(NVR_ERR_UNSUPPORTED, "layer %zu: this feed-forward does not belong to the streams layout", i);
        max_nmix = std::max(max_nmix, w.nmix); max_hv = std::max(max_hv, hv); max_gv = std::max(max_gv, vn);
    }
    RC(named(&embed, (size_t)(V * W * esz))); RC(named(&head, (size_t)(V * W * esz))); RC(own(&wfinal, (size_t)W * 4));
    if (dec_ws_bytes) { RC(own((char **)&dec_ws, dec_ws_bytes)); dec_tickets_n = max_pairs; RC(own(&dec_tickets, (size_t)max_pairs * 4)); }

    // pages for every layer: rotated, normed keys and mixed values
    size_t block_bytes = 0;
    for (const LayeredSpec::Layer &L : spec.layers) block_bytes += (size_t)(r.block_size * L.kv_heads * (L.dim + L.vdim) * esz);
    if (r.cfg.num_kvcache_blocks >= 0) r.num_blocks = r.cfg.num_kvcache_blocks;
    else if (r.cfg.num_kvcache_blocks == -1) r.num_blocks = 1000;
    else {
        size_t free_b = 0, total_b = 0;
        NVR_HIP_CHECK(hipMemGetInfo(&free_b, &total_b));
        const double act_b = (double)MT * (double)(S * W + 6 * W + max_nmix + max_hv + max_gv + 3 * max_ff + max_e2f + max_ef + 3 * max_top * W) * 4.0;
        const int64_t nb = (int64_t)(((double)free_b - (1.0 - r.cfg.gpu_memory_utilization) * (double)total_b - act_b) * 0.9 / (double)block_bytes);
        if (nb < 1) return fail(NVR_ERR_HIP, "not enough free HBM for one KV block");
        r.num_blocks = nb;
    }
    rs.resize(spec.layers.size());
    for (size_t i = 0; i < spec.layers.size(); ++i) {
        const LayeredSpec::Layer &L = spec.layers[i];
        RC(named(&rs[i].kc, (size_t)(r.num_blocks * r.block_size * L.kv_heads * L.dim * esz))); RC(named(&rs[i].vc, (size_t)(r.num_blocks * r.block_size * L.kv_heads * L.vdim * esz)));
    }

    // activations
    RC(named((void **)&x, (size_t)(MT * S * W * 4)));
    RC(named(&a1, (size_t)(MT * W * esz))); RC(named(&a2, (size_t)(MT * W * esz))); RC(named(&tmp, (size_t)(MT * W * esz)));
    RC(named(&proj, (size_t)(MT * max_nmix * esz))); RC(named(&cat, (size_t)(MT * max_hv * esz))); RC(own((char **)&v_first, (size_t)(MT * max_gv * esz)));
    RC(named(&gu, (size_t)(MT * 2 * max_ff * esz))); RC(own((char **)&act, (size_t)(MT * max_ff * esz)));
    const int64_t rows_e = MT * std::max<int64_t>(max_top, 1), pad_rows = (max_experts + 1) * 256;     // (experts' rows padded to whole blocks of 256)
    RC(own((char **)&e_gu, (size_t)(MT * max_e2f * esz))); RC(own((char **)&e_act, (size_t)((MT * max_ef + pad_rows * max_f) * esz)));
    if (max_experts) {
        RC(own((char **)&e_y, (size_t)((rows_e + pad_rows) * W * esz))); RC(own((char **)&e_x, (size_t)((rows_e + pad_rows) * W * esz)));
        RC(own(&rlogits, (size_t)(MT * pad16(max_router)) * 4));
        RC(own(&moe_i, (size_t)(3 * rows_e + max_experts + 1 + rows_e / 256 + max_experts + 1024 + 8) * 4)); RC(own(&moe_score, (size_t)rows_e * 4));
        std::vector<float> one((size_t)rows_e, 1.0f);       // the experts' inputs are the rows as they are: a scale of one per (token, choice)
        RC(own(&gfloor, one.size() * 4)); NVR_HIP_CHECK(hipMemcpy(gfloor, one.data(), one.size() * 4, hipMemcpyHostToDevice));
    }
    return NVR_OK;
}

// Tensors by the names of the checkpoint: "embed", "head", "final.norm" [W]; per layer i "l<i>.norm1" / "norm2" [W], "l<i>.hc1.*" / "l<i>.hc2.*" {in, out} [S], mix [S][S],
// "l<i>.mix.{q,k,v}" with biases "l<i>.mix.{q,k,v}.b", "l<i>.mix.{g,o}", "l<i>.mix.vmix" (one number), "l<i>.mlp.{gate,up,down}" or "l<i>.mlp.{router,correction,e<j>.{gate,up,down}}".
// Linear weights are [out][in].
int LayeredModel::load_streams(nvr_model_runner &r, const std::string &name, int dtype, const int64_t *shape, int ndim, const void *data) {
    const int64_t W = spec.width, V = spec.vocab, S = spec.streams, nL = (int64_t)spec.layers.size();
    const char *name_in = name.c_str();
    auto is2 = [&](int64_t a, int64_t b) { return ndim == 2 && shape[0] == a && shape[1] == b; };
    auto bad = [&]() { return fail(NVR_ERR_LEN_MISMATCH, "load_tensor: '%s' has the wrong shape", name_in); };
    auto unknown = [&]() { return fail(NVR_ERR_UNSUPPORTED, "load_tensor: unknown tensor '%s'", name_in); };
    auto vec = [&](float *dst, int64_t n) { return (dst && ndim == 1 && shape[0] == n) ? put(r, dst, n, 1, n, dtype, data, false) : bad(); };
    auto mat = [&](void *dst, int64_t ld, int64_t rows, int64_t cols) { return (dst && is2(rows, cols)) ? put(r, dst, ld, rows, cols, dtype, data, true) : bad(); };
    auto scalar = [&](float *dst) { int64_t n = 1; for (int i = 0; i < ndim; ++i) n *= shape[i]; return n == 1 ? put(r, dst, 1, 1, 1, dtype, data, false) : bad(); };
    auto rows_at = [&](void *base, int64_t row0, int64_t ld) { return (void *)((char *)base + (size_t)(row0 * ld * esz)); };
    auto number = [](const std::string &t, size_t from, size_t to, int64_t &n) {       // decimal digits [from, to)
        if (from >= to || to - from > 9) return false;
        n = 0;
        for (size_t i = from; i < to; ++i) { if (t[i] < '0' || t[i] > '9') return false; n = n * 10 + (t[i] - '0'); }
        return true;
    };
    if (name == "embed") return mat(embed, W, V, W);
    if (name == "head") return mat(head, W, V, W);
    if (name == "final.norm") return vec(wfinal, W);
    const size_t dot = name.find('.');
    int64_t li = 0;
    if (name.empty() || name[0] != 'l' || dot == std::string::npos || !number(name, 1, dot, li)) return unknown();
    if (li >= nL) return fail(NVR_ERR_UNSUPPORTED, "load_tensor: '%s' names a layer the model does not have", name_in);
    const LayeredSpec::Layer &L = spec.layers[(size_t)li]; LayerW &w = lw[(size_t)li];
    const std::string rest = name.substr(dot + 1);
    const int64_t hd = L.heads * L.dim, kn = L.kv_heads * L.dim, vn = L.kv_heads * L.vdim, hv = L.heads * L.vdim;
    if (rest == "norm1") return vec(w.n1, W);
    if (rest == "norm2" && L.has_mlp) return vec(w.n2, W);
    for (int q = 0; q < (L.has_mlp ? 2 : 1); ++q) {
        const std::string p = q ? "hc2." : "hc1.";
        if (rest == p + "in") return vec(w.hin[q], S);
        if (rest == p + "out") return vec(w.hout[q], S);
        if (rest == p + "mix") return is2(S, S) ? put(r, w.hmix[q], S, S, S, dtype, data, false) : bad();
    }
    if (rest == "mix.q") return mat(rows_at(w.mix, w.qcol, W), W, hd, W);
    if (rest == "mix.k") return mat(rows_at(w.mix, w.kcol, W), W, kn, W);
    if (rest == "mix.v") return mat(rows_at(w.mix, w.vcol, W), W, vn, W);
    if (rest == "mix.g") return mat(rows_at(w.mix, w.gcol, W), W, hv, W);
    if (rest == "mix.o") return mat(w.wo, hv, W, hv);
    if (rest == "mix.q.b") return vec(w.bq, hd);
    if (rest == "mix.k.b") return vec(w.bk, kn);
    if (rest == "mix.v.b") return vec(w.bv, vn);
    if (rest == "mix.vmix") return scalar(w.vmix);              // (read only where the layer mixes)
    if (L.ff_kind == LayeredSpec::FF_GEGLU) {
        if (rest == "mlp.gate") return mat(w.up, W, L.ff, W);
        if (rest == "mlp.up") return mat(rows_at(w.up, L.ff, W), W, L.ff, W);
        if (rest == "mlp.down") return mat(w.down, L.ff, W, L.ff);
    } else if (L.ff_kind == LayeredSpec::FF_MOE_IDENT) {
        const int64_t f = L.expert_ff, ne = L.experts + L.identity;
        if (rest == "mlp.router") return mat(w.router_op, W, ne, W);
        if (rest == "mlp.correction") return vec(w.ecorr, ne);
        const size_t d2 = rest.find('.', 5);
        int64_t e = 0;
        if (rest.compare(0, 5, "mlp.e") == 0 && d2 != std::string::npos && number(rest, 5, d2, e)) {
            if (e >= L.experts) return fail(NVR_ERR_UNSUPPORTED, "load_tensor: '%s' names an expert the layer does not have", name_in);
            const std::string part = rest.substr(d2 + 1);
            if (part == "gate") return mat(rows_at(w.egu, e * 2 * f, W), W, f, W);
            if (part == "up") return mat(rows_at(w.egu, e * 2 * f + f, W), W, f, W);
            if (part == "down") return mat(rows_at(w.edown, e * W, f), f, W, f);
        }
    }
    return unknown();
}

int LayeredModel::forward_streams(nvr_model_runner &r, const StepPlan &p) {
    const kl::Batch &b = p.b;
    const int64_t T = p.T, R = p.R, W = spec.width, nL = (int64_t)spec.layers.size(), MT = r.max_tokens;
    const float eps = (float)spec.eps;
    hipStream_t s = r.stream;
    auto at = [&](void *base, int64_t col) { return (void *)((char *)base + (size_t)(col * esz)); };
    kl::StreamArgs st{}; st.x = x; st.S = (int32_t)spec.streams; st.W = (int32_t)W; st.T = T; st.eps = eps; st.ldy = W; st.ldo = W; st.y = tmp;
    {
        kl::StreamArgs g = st; g.E = embed; g.ids = b.ids; g.win = lw[0].hin[0]; g.w = lw[0].n1; g.out = a1;
        RC(kl::stream_step(g, bf16, s));
    }
    // the end of sublayer q of layer i: its result (tmp) joins the streams; the next sublayer's input leaves in the same pass, or, behind the last one, the logits' rows
    auto join = [&](int64_t i, int q) -> int {
        const LayerW &w = lw[(size_t)i];
        kl::StreamArgs j = st; j.mix = w.hmix[q]; j.wout = w.hout[q];
        if (q == 0 && spec.layers[(size_t)i].has_mlp) { j.win = w.hin[1]; j.w = w.n2; j.out = a2; }
        else if (i + 1 < nL) { j.win = lw[(size_t)(i + 1)].hin[0]; j.w = lw[(size_t)(i + 1)].n1; j.out = a1; }
        else { j.sum = true; j.rows = p.d_want; j.T = R; j.w = wfinal; j.out = xsel; }
        return kl::stream_step(j, bf16, s);
    };
    bool first = true;                                       // no layer has kept its values yet
    for (int64_t i = 0; i < nL; ++i) {
        const LayeredSpec::Layer &L = spec.layers[(size_t)i]; const LayerW &w = lw[(size_t)i]; RunState &rst = rs[(size_t)i];
        const int64_t hv = L.heads * L.vdim, g = L.heads / L.kv_heads;
        RC(gemm(r, a1, W, w.mix, T, W, w.nmix, proj));
        kl::SinkAttnArgs a{};
        a.q = at(proj, w.qcol); a.ldq = w.nmix; a.kc = rst.kc; a.vc = rst.vc; a.H = (int32_t)L.heads; a.G = (int32_t)L.kv_heads; a.D = (int32_t)L.dim; a.Dv = (int32_t)L.vdim;
        a.scale = (float)L.scale; a.out = cat; a.ldo = hv;
        a.v_grouped = w.flash ? 0 : 1;                       // (a property of the layer: the pages keep one layout)
        const bool tiled = kl::sink_attention_tiled_ok(a, bf16, (int)r.block_size);
        kl::QkvRopeArgs qa{};
        qa.proj = proj; qa.ld = w.nmix; qa.qcol = w.qcol; qa.kcol = w.kcol; qa.vcol = w.vcol; qa.H = a.H; qa.G = a.G; qa.D = a.D; qa.Dv = a.Dv;
        qa.rot = (int32_t)L.rot_dims; qa.freq = w.rfreq; qa.pairs = true; qa.bq = w.bq; qa.bk = w.bk; qa.bv = w.bv; qa.unit = true; qa.eps = eps;
        if (L.v_mix) { if (first) qa.v_keep = v_first; else { qa.v_first = v_first; qa.lambda = w.vmix; } first = false; }
        qa.kc = rst.kc; qa.vc = rst.vc; qa.v_grouped = tiled && !w.flash;
        RC(kl::qkv_rope_store(qa, b, bf16, s));
        if (w.flash && p.decode_sized) {
            nvr::kt::AttnArgs d{};
            d.q = (const uint16_t *)a.q; d.ldq = w.nmix; d.k = (const uint16_t *)rst.kc; d.v = (const uint16_t *)rst.vc; d.ctx_lens = p.d_ctx;
            d.block_tables = b.block_tables; d.max_blocks = b.max_blocks; d.block_size = b.block_size; d.nq = (int32_t)T; d.H = a.H; d.KVH = a.G; d.D = a.D;
            d.scale = a.scale; d.max_ctx = (int32_t)p.max_ctx; d.out = (uint16_t *)cat; d.workspace = dec_ws; d.workspace_bytes = dec_ws_bytes; d.tickets = dec_tickets;
            RC(nvr::kb::attention(d, true, s));
        } else if (w.flash) {
            const size_t gi = flash_kind(nvr::kb::flash_tile_positions((int)L.heads, (int)L.kv_heads));
            nvr::kt::FlashArgs f{};
            f.q = (const uint16_t *)a.q; f.ldq = w.nmix; f.k = (const uint16_t *)rst.kc; f.v = (const uint16_t *)rst.vc; f.ldkv = 0;
            f.block_tables = b.block_tables; f.max_blocks = b.max_blocks; f.block_size = b.block_size;
            f.tiles = (const nvr::kt::FlashTile *)(in_dev + p.o_ftiles[gi]); f.ntiles = p.n_ftiles[gi];
            f.H = a.H; f.KVH = a.G; f.D = a.D; f.scale = a.scale; f.out = (uint16_t *)cat; f.ldo = hv;
            RC(nvr::kb::flash_prefill(f, true, s));
        } else if (tiled) {
            const size_t gi = index_of(attn_groups, g);
            // decode-sized steps over long contexts: few tiles, many keys each — a tile's keys go to several workgroups
            const int64_t wgs = (int64_t)p.n_tiles[gi] * L.kv_heads;
            int64_t nsplit = 1;
            if (wgs < r.num_cus && p.max_ctx >= 512) nsplit = std::max<int64_t>(1, std::min<int64_t>({(2 * r.num_cus) / wgs, (p.max_ctx + 255) / 256, 16}));
            RC(kl::sink_attention_tiled(a, b, (const kl::AttnTile *)(in_dev + p.o_tiles[gi]), p.n_tiles[gi], (int)nsplit, attn_ws, attn_ws_bytes, s));
        } else
            RC(kl::sink_attention(a, b, bf16, s));
        RC(kl::sigmoid_gate(cat, hv, at(proj, w.gcol), w.nmix, T, hv, bf16, s));
        RC(gemm(r, cat, hv, w.wo, T, hv, W, tmp));
        RC(join(i, 0));
        if (L.ff_kind == LayeredSpec::FF_GEGLU) {
            if (bf16 && W % 32 == 0 && L.ff % 16 == 0) RC(nvr::kb::linear_gelu_mul((const uint16_t *)a2, W, (const uint16_t *)w.up, T, W, L.ff, (uint16_t *)act, s));   // (gate, up and GELU in one launch)
            else {
                RC(gemm(r, a2, W, w.up, T, W, 2 * L.ff, gu));
                RC(kl::gelu_mul(gu, T, L.ff, act, L.ff, bf16, s));
            }
            RC(gemm(r, act, L.ff, w.down, T, L.ff, W, tmp));
        } else if (L.ff_kind == LayeredSpec::FF_MOE_IDENT) {
            const int64_t f = L.expert_ff, n = T * L.top, ne = pad16(L.experts + L.identity);
            int32_t *sel = moe_i, *order = sel + MT * L.top, *place_of = order + MT * L.top, *off = place_of + MT * L.top, *row_w = off + L.experts + 1;
            // many rows: every expert's rows padded to whole blocks of 256, brought together once, and the dense graph's 256 x 256 product with a matrix per row block
            const int64_t nblocks = n / 256 + L.experts;
            const bool blocks = bf16 && n >= 2048 && nvr::kb::gemm256_silu_ok(nblocks * 256, W, f, W) && nvr::kb::gemm256_ok(nblocks * 256, f, W, f);
            RC(gemm(r, a2, W, w.router_op, T, W, ne, rlogits, true));                  // router logits: f32 accumulation, f32 output
            RC(kl::moe_route(a2, W, T, W, nullptr, L.experts + L.identity, L.top, sel, moe_score, off, order, place_of, blocks ? 256 : 1, blocks ? row_w : nullptr, nblocks, bf16, s,
                             true, 0, nullptr, rlogits, ne, w.ecorr, L.identity));
            if (blocks) {
                RC(kl::moe_gather(a2, W, T, W, L.top, place_of, gfloor, e_x, bf16, s));
                RC(nvr::kb::gemm256_grouped_silu_mul((const uint16_t *)e_x, W, (const uint16_t *)w.egu, 2 * f * W, row_w, nblocks * 256, W, f, (uint16_t *)e_act, s, off + L.experts));
                RC(nvr::kb::gemm256_grouped((const uint16_t *)e_act, f, (const uint16_t *)w.edown, W * f, row_w, nblocks * 256, f, W, (uint16_t *)e_y, s, off + L.experts));
            } else {
                kl::GroupedLinearArgs gl{}; gl.a = a2; gl.lda = W; gl.w = w.egu; gl.y = e_gu; gl.ldy = 2 * f; gl.off = off; gl.groups = (int32_t)L.experts; gl.K = (int32_t)W; gl.N = (int32_t)(2 * f);
                gl.max_rows = (int32_t)n; gl.src = order; gl.rscale = gfloor; gl.src_div = (int32_t)L.top;
                RC(kl::grouped_linear(gl, bf16, s));
                RC(kl::silu_mul(e_gu, n, f, e_act, f, bf16, s));
                kl::GroupedLinearArgs d{}; d.a = e_act; d.lda = f; d.w = w.edown; d.y = e_y; d.ldy = W; d.off = off; d.groups = (int32_t)L.experts; d.K = (int32_t)f; d.N = (int32_t)W; d.max_rows = (int32_t)n;
                RC(kl::grouped_linear(d, bf16, s));
            }
            st.place = place_of; st.top = (int32_t)L.top; st.score = moe_score; st.ident = a2; st.ldi = W; st.y = e_y;      // (the choices' rows are summed up where they join the streams)
        }
        if (L.has_mlp) { RC(join(i, 1)); st.place = nullptr; st.y = tmp; }
    }
    return gemm(r, xsel, W, head, R, W, spec.vocab, r.logits, true);
}

}  // namespace nvr
