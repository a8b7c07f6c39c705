// Layer-stack decoders: a model described layer by layer (include/llava_mi355x.h: lmx_stack_config / lmx_layer_config) on the engine's own sequences, caches, decode
// batches, samplers and linears.  What differs from the LLaMA decoder of engine.cpp:
//
//   * the residual stream is fp32 in every model dtype; a sublayer's output may be normalised before it is added (times residual_mult), so no linear adds a residual in its
//     epilogue — residual_norm (stack_ops.hip) does post-norm, addition and the next sublayer's pre-norm in one launch between any two linears;
//   * a range of layers may run several times in a row (loop): weights exist once per LAYER, caches and states once per layer RUN; before each pass but the first the
//     embedding row is added to the residual (inject), in the launch that ends the previous layer, or before every pass x <- W [x; embedding row] (mix);
//   * per layer: the mixer (softmax attention here; latent attention and the gated delta rule in stack_mixers.cpp), its head counts and widths and options, the
//     feed-forward (none, gated, a mixture of gated experts), and whether the two follow each other or both read one norm (parallel);
//   * an embedding row may depend on the token before (bigram): input rows are then ids, and the last token is part of a sequence's state;
//   * logits are fp32 and soft-capped in the lm_head's epilogue.
//
// Layout: width and ff are padded to multiples of 64, head vectors to D in {64, 128, 256}, the vocabulary to 8, all with zero weights, so that padded lanes stay zero
// through every op (norm means divide by the true sizes).  One fused weight per layer for everything the mixer projects from the normed row; gate | up interleaved as in
// the LLaMA decoder; a parallel layer's dense down projection sits beside the output projection (one product over mixer row | activations).
#include "engine.h"

#include <cstring>

namespace lmx {

static int round_up(int a, int b) { return (a + b - 1) / b * b; }

Model::Model(const lmx_stack_config& c, const lmx_layer_config* layers) {
    LMX_REQUIRE(c.abi_version == LMX_ABI_VERSION, "lmx_stack_config.abi_version mismatch");
    LMX_REQUIRE(c.dtype == kF32 || c.dtype == kBF16 || c.dtype == kF16, "bad dtype");
    LMX_REQUIRE(c.width >= 1 && c.vocab_size >= 1 && c.n_layers >= 1 && layers, "stack: empty model");
    LMX_REQUIRE(c.loop_times >= 1 && c.loop_start >= 0 && c.loop_start <= c.loop_stop && c.loop_stop <= c.n_layers, "stack: bad loop range");
    cfg.abi_version = c.abi_version; cfg.dtype = c.dtype; cfg.hidden_size = c.width; cfg.vocab_size = c.vocab_size; cfg.n_layers = c.n_layers;
    cfg.rms_eps = c.norm_eps; cfg.max_position = c.max_position; cfg.tp_world = 1; cfg.tp_rank = 0; cfg.gemm_variant = c.gemm_variant;
    es = (int)dtype_size(c.dtype);
    stk = std::make_unique<Stack>();
    Stack& S = *stk;
    S.c = c;
    H = round_up(c.width, 64);
    LMX_REQUIRE(H <= 8192, "stack: width up to 8192");
    V = round_up(c.vocab_size, 8); Vr = c.vocab_size; V_l = V; v_off = 0;
    les = 4;
    s_max = round_up(c.max_position > 0 ? c.max_position : 2048, 128);
    S.layers.resize((size_t)c.n_layers);
    for (int i = 0; i < c.n_layers; ++i) {
        StackLayer& l = S.layers[(size_t)i];
        const lmx_layer_config& d = l.c = layers[i];
        LMX_REQUIRE(d.mixer >= LMX_MIXER_ATTENTION && d.mixer <= LMX_MIXER_DELTA, "stack: unknown mixer");
        LMX_REQUIRE(d.n_heads >= 1 && d.n_kv_heads >= 1 && d.n_heads % d.n_kv_heads == 0, "stack: n_heads must be a multiple of n_kv_heads");
        LMX_REQUIRE(d.qk_dim >= 1 && d.v_dim >= 1 && d.qk_dim <= 256 && d.v_dim <= 256, "stack: head widths up to 256");
        LMX_REQUIRE(d.rope_dims >= 0 && d.rope_dims % 2 == 0 && d.rope_dims <= d.qk_dim, "stack: rotated dimensions must be even and inside the head");
        LMX_REQUIRE(d.rope_dims == 0 || (d.rope_table >= 0 && d.rope_table < 256), "stack: bad rope table index");
        LMX_REQUIRE(d.window >= 0 && d.ff >= 0, "stack: bad window / feed-forward width");
        const int m = std::max(d.qk_dim, d.v_dim);
        l.D = m <= 64 ? 64 : m <= 128 ? 128 : 256;
        l.an = d.n_heads * l.D;
        l.ff = round_up(d.ff, 64);
        LMX_REQUIRE(d.ff_act == 0 || d.ff_act == LMX_ACT_SILU_MUL || d.ff_act == LMX_ACT_RELU_MUL, "stack: unknown feed-forward activation");
        LMX_REQUIRE(d.experts == 0 || (d.ff > 0 && d.experts <= 256 && d.top_experts >= 1 && d.top_experts <= std::min(d.experts, 32)), "stack: 1..256 experts, at most 32 of them per row");
        if (d.mixer == LMX_MIXER_LATENT) {
            LMX_REQUIRE(d.q_rank >= 1 && d.kv_rank >= 1 && d.kv_rank <= 512 && d.rope_dims == 0, "stack: latent attention needs its ranks (kv_rank up to 512) and has no positions");
            l.Q = round_up(d.q_rank, 64);
            l.R = d.kv_rank <= 64 ? 64 : d.kv_rank <= 128 ? 128 : d.kv_rank <= 256 ? 256 : 512;
            l.qkv_n = l.Q + l.R;
            S.q_n = std::max(S.q_n, l.an); S.lat_n = std::max(S.lat_n, d.n_heads * l.R);
            S.dec_ws = std::max(S.dec_ws, decode_fused_ws_floats(d.n_heads, 32, l.R));
        } else if (d.mixer == LMX_MIXER_DELTA) {
            LMX_REQUIRE(d.conv_taps >= 1 && d.decay_rank >= 1 && d.gate_rank >= 1, "stack: the delta rule needs its taps and inner widths");
            l.ds = DeltaShape{d.n_heads, d.n_kv_heads, d.qk_dim <= 64 ? 64 : d.qk_dim <= 128 ? 128 : 256, round_up(d.v_dim, 64), d.qk_dim, d.v_dim, d.conv_taps};
            l.ra = round_up(d.decay_rank, 64); l.rg = round_up(d.gate_rank, 64);
            l.an = l.ds.H * l.ds.DV;
            l.qkv_n = l.a_off() + l.ra + l.rg;
        } else {
            l.gate_off = d.out_gate ? (d.n_heads + 2 * d.n_kv_heads) * l.D : -1;
            l.qkv_n = (d.n_heads + 2 * d.n_kv_heads) * l.D + (d.out_gate ? round_up(d.n_heads, 64) : 0);
        }
        l.out_k = l.an + (l.parallel() && l.dense() ? l.ff : 0);
        if (l.moe()) { S.moe_act = std::max(S.moe_act, d.top_experts * l.ff); S.moe_top = std::max(S.moe_top, d.top_experts); }
        if (d.rope_dims && d.rope_table >= (int)S.rope.size()) { S.rope.resize((size_t)d.rope_table + 1, nullptr); S.rope_dims.resize((size_t)d.rope_table + 1, 0); }
        // sizes the shared workspaces (Seq, Batch) are cut by: the widest layer
        D = std::max(D, l.D); nh_l = std::max(nh_l, d.n_heads); nkv_l = std::max(nkv_l, d.n_kv_heads);
        qkv_n = std::max(qkv_n, l.qkv_n); I_l = std::max(I_l, std::max(l.ff, 64)); S.mix_n = std::max(S.mix_n, l.out_k);
        S.dec_ws = std::max(S.dec_ws, decode_fused_ws_floats(d.n_heads, std::min((s_max + 127) / 128, 32), l.D));
    }
    LMX_REQUIRE(c.bigram_buckets >= 0 && (c.bigram_buckets == 0 || c.loop_mix || c.loop_times == 1), "stack: rows that come as ids cannot be added again before a pass");
    auto run = [&](int layer, bool begins, int pass) {
        const StackLayer& l = S.layers[(size_t)layer];
        auto up = [](size_t b) { return (b + 255) / 256 * 256; };
        StackRun r{layer, begins && !c.loop_mix && pass > 0, begins && c.loop_mix != 0, S.k_bytes, S.v_bytes, S.s_bytes, 0};
        if (l.c.mixer == LMX_MIXER_ATTENTION) {
            const size_t bytes = up((size_t)l.c.n_kv_heads * s_max * l.D * es);
            S.k_bytes += bytes; S.v_bytes += bytes;
        } else if (l.c.mixer == LMX_MIXER_LATENT) S.k_bytes += up((size_t)s_max * l.R * es);
        else {
            r.r_off = r.s_off + up(l.ds.state_floats() * 4);
            S.s_bytes = r.r_off + up((size_t)l.ds.taps * l.ds.channels() * es);
        }
        S.runs.push_back(r);
    };
    for (int i = 0; i < c.loop_start; ++i) run(i, false, 0);
    for (int t = 0; t < c.loop_times; ++t)
        for (int i = c.loop_start; i < c.loop_stop; ++i) run(i, i == c.loop_start, t);
    for (int i = c.loop_stop; i < c.n_layers; ++i) run(i, false, 0);
    L = (int)S.runs.size();
    LMX_REQUIRE(L >= 1, "stack: no layer runs");
    LMX_CHECK_HIP(hipEventCreateWithFlags(&vws_done, hipEventDisableTiming));
}

void Model::stack_set_rope(int table, int dims, const float* host, int n_pos) {
    LMX_REQUIRE(stk, "not a layer-stack model");
    LMX_REQUIRE(table >= 0 && table < (int)stk->rope.size() && dims > 0 && host && n_pos >= s_max, "rope table: bad index or too few positions");
    float*& p = stk->rope[(size_t)table];
    if (p) { (void)hipFree(p); p = nullptr; }
    LMX_CHECK_HIP(hipMalloc(reinterpret_cast<void**>(&p), (size_t)n_pos * dims * sizeof(float)));
    LMX_CHECK_HIP(hipMemcpy(p, host, (size_t)n_pos * dims * sizeof(float), hipMemcpyHostToDevice));
    stk->rope_dims[(size_t)table] = dims;
}

// ---------------------------------------------------------------------------------------------------------------
// weights.  Names: embed, head, bigram, loop.in, final.norm, and per layer l<i>.{norm1, norm1b, norm2, norm2b, mix.*, mlp.*} with
//   attention  mix.{q, k, v}[.b], mix.{q, k}.norm, mix.g, mix.o            latent  mix.{dq, uq, dkv, uk, uv, o}, mix.{dq, dkv}.norm
//   delta      mix.{q, k, v}[.conv], mix.{b, A_log, a1, a2, dt_bias, g1, g2, norm, o}
//   mlp.{gate, up, down}, or mlp.e<j>.{gate, up, down} and mlp.router[.b]
// ---------------------------------------------------------------------------------------------------------------
void Model::stack_load_weight(const std::string& name, const void* src, int ndim, const int64_t* shape, hipStream_t st) {
    Stack& S = *stk;
    const int W = S.c.width, dt = cfg.dtype;
    auto expect = [&](std::initializer_list<int64_t> want) {
        bool ok = (int)want.size() == ndim;
        int i = 0;
        for (auto w : want) { if (ok && shape[i] != w) ok = false; ++i; }
        if (ok) return;
        std::string got = "[", exp = "[";
        for (int k = 0; k < ndim; ++k) got += std::to_string(shape[k]) + ",";
        for (auto w : want) exp += std::to_string(w) + ",";
        throw Error{"shape mismatch for " + name + ": got " + got + "] expected " + exp + "]"};
    };
    // rows [0, rows) x cols of a [rows][cols] source into dst (pitch dst_cols) at (row0, col0)
    auto block = [&](void* dst, int dst_cols, int row0, int col0, const void* s, int src_cols, int rows, int cols) {
        LMX_CHECK_HIP(hipMemcpy2DAsync(static_cast<char*>(dst) + ((size_t)row0 * dst_cols + col0) * es, (size_t)dst_cols * es, s, (size_t)src_cols * es, (size_t)cols * es,
                                       (size_t)rows, hipMemcpyDeviceToDevice, st));
    };
    auto at = [&](size_t elems) { return static_cast<const char*>(src) + elems * es; };
    auto vec = [&](void*& dst, int n, int padded) {
        expect({n});
        if (!dst) dst = alloc_weight((size_t)padded * es, true);
        block(dst, padded, 0, 0, src, n, 1, n);
    };
    auto table = [&](void*& dst) {
        expect({S.c.vocab_size, W});
        if (!dst) dst = alloc_weight((size_t)V * H * es, true);
        block(dst, H, 0, 0, src, W, S.c.vocab_size, W);
    };
    if (name == "embed") table(embed);
    else if (name == "head" && !S.c.tied_head) table(lm_head);
    else if (name == "bigram" && S.ids_in()) {
        expect({(int64_t)S.c.bigram_buckets + 1, W});
        if (!S.bigram) S.bigram = alloc_weight((size_t)(S.c.bigram_buckets + 1) * H * es, true);
        block(S.bigram, H, 0, 0, src, W, S.c.bigram_buckets + 1, W);
    }
    else if (name == "loop.in" && S.c.loop_mix) {
        expect({W, 2 * (int64_t)W});
        if (!S.loop_in) S.loop_in = alloc_weight((size_t)H * 2 * H * es, true);
        block(S.loop_in, 2 * H, 0, 0, src, 2 * W, W, W);
        block(S.loop_in, 2 * H, 0, H, at((size_t)W), 2 * W, W, W);
    }
    else if (name == "final.norm") vec(final_norm, W, H);
    else {
        const size_t dot = name.find('.');
        LMX_REQUIRE(name.size() > 2 && name[0] == 'l' && dot != std::string::npos && dot > 1, "unknown tensor name: " + name);
        for (size_t k = 1; k < dot; ++k) LMX_REQUIRE(name[k] >= '0' && name[k] <= '9', "unknown tensor name: " + name);
        const int li = atoi(name.substr(1, dot - 1).c_str());
        LMX_REQUIRE(li >= 0 && li < S.c.n_layers, "layer index out of range: " + name);
        const std::string sub = name.substr(dot + 1);
        StackLayer& l = S.layers[(size_t)li];
        const lmx_layer_config& d = l.c;
        if (!l.wqkv) {
            l.wqkv = alloc_weight((size_t)l.qkv_n * H * es, true);
            if (d.qkv_bias) l.bqkv = alloc_weight((size_t)l.qkv_n * es, true);
            l.wo = alloc_weight((size_t)H * l.out_k * es, true);
            const size_t ne = (size_t)std::max(1, d.experts);
            if (l.ff) l.wgu = alloc_weight(ne * 2 * l.ff * H * es, true);
            if (l.ff && l.out_k == l.an) l.wd = alloc_weight(ne * H * l.ff * es, true);
            if (l.moe()) { l.wr = alloc_weight((size_t)d.experts * H * es, true); l.br = alloc_weight((size_t)d.experts * es, true); }
            if (d.mixer == LMX_MIXER_LATENT) {
                l.wuq = alloc_weight((size_t)l.an * l.Q * es, true);
                l.wukv = alloc_weight((size_t)2 * l.an * l.R * es, true);
                l.wuk_t = alloc_weight((size_t)l.an * l.R * es, true);
            } else if (d.mixer == LMX_MIXER_DELTA) {
                l.conv = alloc_weight((size_t)l.ds.taps * l.ds.channels() * es, true);
                l.dt_bias = alloc_weight((size_t)l.ds.H * l.ds.DK * es, true);
                l.wag = alloc_weight((size_t)l.ds.H * (l.ds.DK + l.ds.DV) * (l.ra + l.rg) * es, true);
            }
        }
        auto head_rows = [&](void* dst, int dst_cols, int row0, int col0, int n, int dim, int padded, int cols) {      // [n * dim][cols] -> blocks of `padded` rows
            expect({(int64_t)n * dim, cols});
            for (int h = 0; h < n; ++h) block(dst, dst_cols, row0 + h * padded, col0, at((size_t)h * dim * cols), cols, dim, cols);
        };
        auto rows_at = [&](int row0, int n) { expect({n, W}); block(l.wqkv, H, row0, 0, src, W, n, W); };
        auto heads = [&](int first_slot, int n, int dim) {                    // [n * dim][W] -> one padded head block per head
            expect({(int64_t)n * dim, W});
            for (int h = 0; h < n; ++h) block(l.wqkv, H, (first_slot + h) * l.D, 0, at((size_t)h * dim * W), W, dim, W);
        };
        auto head_bias = [&](int first_slot, int n, int dim) {
            LMX_REQUIRE(d.qkv_bias, "projection bias given but the layer has none: " + name);
            expect({(int64_t)n * dim});
            block(l.bqkv, l.D, first_slot, 0, src, dim, n, dim);
        };
        auto gate_up = [&](int half, int expert = 0) {
            LMX_REQUIRE(d.ff > 0, "feed-forward tensor given but the layer has none: " + name);
            expect({d.ff, W});
            void* wgu = static_cast<char*>(l.wgu) + (size_t)expert * 2 * l.ff * H * es;
            DevBuf tmp;                                                       // rows padded to whole 32-row groups and columns to the padded width
            tmp.ensure((size_t)l.ff * H * es, true);
            block(tmp.p, H, 0, 0, src, W, d.ff, W);
            launch_interleave_half(dt, tmp.p, wgu, l.ff, H, half, st);
            LMX_CHECK_HIP(hipStreamSynchronize(st));
        };
        auto down = [&](int expert) {
            expect({W, d.ff});
            if (l.out_k > l.an) block(l.wo, l.out_k, 0, l.an, src, d.ff, W, d.ff);
            else block(static_cast<char*>(l.wd) + (size_t)expert * H * l.ff * es, l.ff, 0, 0, src, d.ff, W, d.ff);
        };
        const int nh = d.n_heads, nk = d.n_kv_heads;
        const DeltaShape& ds = l.ds;
        // convolution taps [channels][taps] -> [taps][padded channels]
        auto conv = [&](int first, int n, int dim, int padded) {
            expect({(int64_t)n * dim, ds.taps});
            for (int h = 0; h < n; ++h)
                launch_transpose(dt, at((size_t)h * dim * ds.taps), ds.taps, dim, ds.taps, static_cast<char*>(l.conv) + (size_t)(first + h * padded) * es, ds.channels(), st);
        };
        const bool delta = d.mixer == LMX_MIXER_DELTA, lat = d.mixer == LMX_MIXER_LATENT;
        if (sub == "norm1") vec(l.n1, W, H);
        else if (sub == "norm1b" && !l.parallel()) vec(l.n1b, W, H);
        else if ((sub == "norm2" || sub == "norm2b") && !d.ff) return;       // norms of a feed-forward the layer does not have
        else if (sub == "norm2" && !l.parallel()) vec(l.n2, W, H);
        else if (sub == "norm2b" && !l.parallel()) vec(l.n2b, W, H);
        else if (delta && sub == "mix.q") head_rows(l.wqkv, H, 0, 0, nk, d.qk_dim, ds.DK, W);
        else if (delta && sub == "mix.k") head_rows(l.wqkv, H, nk * ds.DK, 0, nk, d.qk_dim, ds.DK, W);
        else if (delta && sub == "mix.v") head_rows(l.wqkv, H, 2 * nk * ds.DK, 0, nh, d.v_dim, ds.DV, W);
        else if (delta && sub == "mix.q.conv") conv(0, nk, d.qk_dim, ds.DK);
        else if (delta && sub == "mix.k.conv") conv(nk * ds.DK, nk, d.qk_dim, ds.DK);
        else if (delta && sub == "mix.v.conv") conv(2 * nk * ds.DK, nh, d.v_dim, ds.DV);
        else if (delta && sub == "mix.b") rows_at(ds.channels(), nh);
        else if (delta && sub == "mix.a1") rows_at(l.a_off(), d.decay_rank);
        else if (delta && sub == "mix.g1") rows_at(l.a_off() + l.ra, d.gate_rank);
        else if (delta && sub == "mix.a2") head_rows(l.wag, l.ra + l.rg, 0, 0, nh, d.qk_dim, ds.DK, d.decay_rank);
        else if (delta && sub == "mix.g2") head_rows(l.wag, l.ra + l.rg, nh * ds.DK, l.ra, nh, d.v_dim, ds.DV, d.gate_rank);
        else if (delta && sub == "mix.A_log") vec(l.a_log, nh, round_up(nh, 8));
        else if (delta && sub == "mix.dt_bias") { expect({(int64_t)nh * d.qk_dim}); block(l.dt_bias, ds.DK, 0, 0, src, d.qk_dim, nh, d.qk_dim); }
        else if (delta && sub == "mix.norm") vec(l.onorm, d.v_dim, ds.DV);
        else if (lat && sub == "mix.dq") rows_at(0, d.q_rank);
        else if (lat && sub == "mix.dkv") rows_at(l.Q, d.kv_rank);
        else if (lat && sub == "mix.dq.norm") vec(l.qn_lat, d.q_rank, l.Q);
        else if (lat && sub == "mix.dkv.norm") vec(l.kn_lat, d.kv_rank, l.R);
        else if (lat && sub == "mix.uq") head_rows(l.wuq, l.Q, 0, 0, nh, d.qk_dim, l.D, d.q_rank);
        else if (lat && sub == "mix.uk") {
            head_rows(l.wukv, l.R, 0, 0, nh, d.qk_dim, l.D, d.kv_rank);
            for (int h = 0; h < nh; ++h)
                launch_transpose(dt, at((size_t)h * d.qk_dim * d.kv_rank), d.kv_rank, d.qk_dim, d.kv_rank, static_cast<char*>(l.wuk_t) + (size_t)h * l.R * l.D * es, l.D, st);
        }
        else if (lat && sub == "mix.uv") head_rows(l.wukv, l.R, nh * l.D, 0, nh, d.v_dim, l.D, d.kv_rank);
        else if (sub == "mix.o") {
            expect({W, (int64_t)nh * d.v_dim});
            const int hp = l.an / nh;
            for (int h = 0; h < nh; ++h) block(l.wo, l.out_k, 0, h * hp, at((size_t)h * d.v_dim), nh * d.v_dim, W, d.v_dim);
        }
        else if (l.moe() && sub == "mlp.router") { expect({d.experts, W}); block(l.wr, H, 0, 0, src, W, d.experts, W); }
        else if (l.moe() && sub == "mlp.router.b") { expect({d.experts}); block(l.br, d.experts, 0, 0, src, d.experts, 1, d.experts); }
        else if (l.moe() && sub.rfind("mlp.e", 0) == 0) {
            const size_t q = sub.find('.', 5);
            LMX_REQUIRE(q != std::string::npos && q > 5 && q <= 9, "unknown tensor name: " + name);
            for (size_t k = 5; k < q; ++k) LMX_REQUIRE(sub[k] >= '0' && sub[k] <= '9', "unknown tensor name: " + name);
            const int ex = atoi(sub.substr(5, q - 5).c_str());
            LMX_REQUIRE(ex >= 0 && ex < d.experts, "expert index out of range: " + name);
            const std::string leaf = sub.substr(q + 1);
            if (leaf == "gate") gate_up(0, ex); else if (leaf == "up") gate_up(1, ex); else if (leaf == "down") down(ex); else throw Error{"unknown tensor name: " + name};
        }
        else if (sub == "mlp.gate" && l.dense()) gate_up(0);
        else if (sub == "mlp.up" && l.dense()) gate_up(1);
        else if (sub == "mlp.down" && l.dense()) down(0);
        else if (delta || lat) throw Error{"unknown tensor name: " + name};
        else if (sub == "mix.q") heads(0, nh, d.qk_dim);
        else if (sub == "mix.k") heads(nh, nk, d.qk_dim);
        else if (sub == "mix.v") heads(nh + nk, nk, d.v_dim);
        else if (sub == "mix.q.b") head_bias(0, nh, d.qk_dim);
        else if (sub == "mix.k.b") head_bias(nh, nk, d.qk_dim);
        else if (sub == "mix.v.b") head_bias(nh + nk, nk, d.v_dim);
        else if (sub == "mix.q.norm" && d.qk_norm) vec(l.qn, d.qk_dim, l.D);
        else if (sub == "mix.k.norm" && d.qk_norm) vec(l.kn, d.qk_dim, l.D);
        else if (sub == "mix.g" && d.out_gate) { expect({nh, W}); block(l.wqkv, H, l.gate_off, 0, src, W, nh, W); }
        else throw Error{"unknown tensor name: " + name};
    }
    loaded.insert(name);
}

void Model::stack_finalize() {
    std::string missing;
    auto need = [&](const std::string& n) { if (!loaded.count(n)) missing += n + " "; };
    need("embed"); need("final.norm");
    if (!stk->c.tied_head) need("head");
    if (stk->ids_in()) need("bigram");
    if (stk->c.loop_mix) need("loop.in");
    for (int i = 0; i < stk->c.n_layers; ++i) {
        const lmx_layer_config& d = stk->layers[(size_t)i].c;
        const std::string p = "l" + std::to_string(i) + ".";
        for (const char* s : {"norm1", "mix.o"}) need(p + s);
        if (!d.parallel) { need(p + "norm1b"); if (d.ff) { need(p + "norm2"); need(p + "norm2b"); } }
        if (d.ff && !d.experts) for (const char* s : {"mlp.gate", "mlp.up", "mlp.down"}) need(p + s);
        if (d.experts) {
            need(p + "mlp.router"); need(p + "mlp.router.b");
            for (int e = 0; e < d.experts; ++e) for (const char* s : {"gate", "up", "down"}) need(p + "mlp.e" + std::to_string(e) + "." + s);
        }
        if (d.mixer == LMX_MIXER_LATENT) { for (const char* s : {"dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv"}) need(p + "mix." + s); continue; }
        if (d.mixer == LMX_MIXER_DELTA) {
            for (const char* s : {"q", "q.conv", "k", "k.conv", "v", "v.conv", "b", "A_log", "norm", "a1", "a2", "dt_bias", "g1", "g2"}) need(p + "mix." + s);
            continue;
        }
        for (const char* s : {"mix.q", "mix.k", "mix.v"}) need(p + s);
        if (d.qkv_bias) for (const char* s : {"mix.q.b", "mix.k.b", "mix.v.b"}) need(p + s);
        if (d.qk_norm) for (const char* s : {"mix.q.norm", "mix.k.norm"}) need(p + s);
        if (d.out_gate) need(p + "mix.g");
        if (d.rope_dims) {
            const bool ok = stk->rope[(size_t)d.rope_table] && stk->rope_dims[(size_t)d.rope_table] == d.rope_dims;
            if (!ok) missing += "<rope table " + std::to_string(d.rope_table) + "> ";
        }
    }
    if (!missing.empty()) throw Error{"missing tensors: " + missing};
    if (stk->c.tied_head) lm_head = embed;
}

void Model::stack_batch_weights(hipStream_t st) {
    auto mk = [&](const void* W, int N, int K) -> void* {
        if (!W) return nullptr;
        void* d = alloc_weight(skinny_swizzled_bytes(N, K, es));
        launch_skinny_swizzle(cfg.dtype, W, K, d, N, K, st);
        return d;
    };
    for (StackLayer& l : stk->layers) {
        l.sw_qkv = mk(l.wqkv, l.qkv_n, H);
        l.sw_o = mk(l.wo, H, l.out_k);
        if (l.dense()) { l.sw_gu = mk(l.wgu, 2 * l.ff, H); l.sw_d = mk(l.wd, H, l.ff); }
        l.sw_uq = mk(l.wuq, l.an, l.Q);
    }
    stk->sw_loop = mk(stk->loop_in, H, 2 * H);
    sw_lm_head = mk(lm_head, V, H);
    LMX_CHECK_HIP(hipStreamSynchronize(st));
}

// what ends sublayer `sub` (0 mixer, 1 feed-forward) of run r: its post-norm, the injected rows if the next run wants them, and the norm in front of the next linear
struct StackStep { const void* post; const void* pre; bool inject, mix; };
static StackStep stack_step(const Stack& S, int r, int sub, const void* final_norm) {
    const StackLayer& l = S.layers[(size_t)S.runs[(size_t)r].layer];
    if (sub == 0 && l.ff && !l.parallel()) return {l.n1b, l.n2, false, false};
    const void* post = l.parallel() ? nullptr : sub == 0 ? l.n1b : l.n2b;
    if (r + 1 == (int)S.runs.size()) return {post, final_norm, false, false};
    const StackRun& nx = S.runs[(size_t)r + 1];
    return {post, S.layers[(size_t)nx.layer].n1, nx.inject, nx.mix};
}

static QkvNormRopeArgs rope_args(const Stack& S, const StackLayer& l, void* qkv, void* kc, void* vt, int T, int pos0, int s_max) {
    const lmx_layer_config& d = l.c;
    return QkvNormRopeArgs{qkv, kc, vt, l.qn, l.kn, d.rope_dims ? S.rope[(size_t)d.rope_table] : nullptr, T, pos0, l.qkv_n, d.n_heads, d.n_kv_heads, s_max, d.qk_dim, d.rope_dims, S.c.norm_eps};
}

// ---------------------------------------------------------------------------------------------------------------
// prefill: one sequence or several packed, as Model::prefill_multi walks them (pieces of block_rows rows; linears over the piece, attention per segment)
// ---------------------------------------------------------------------------------------------------------------
void Model::stack_prefill(Seq* const* seqs, const void* const* embeds, const int* Ts, int n, int block_rows, bool greedy, const StackOutputs& out, hipStream_t st) {
    Stack& S = *stk;
    LMX_REQUIRE(n >= 1 && seqs && embeds && Ts, "prefill: bad arguments");
    long total = 0;
    for (int i = 0; i < n; ++i) {
        LMX_REQUIRE(seqs[i] && seqs[i]->m == this && embeds[i] && Ts[i] > 0, "prefill: bad sequence / input");
        LMX_REQUIRE(seqs[i]->len + Ts[i] <= s_max, "prefill: sequence would exceed the KV-cache capacity (max_position)");
        for (int j = 0; j < i; ++j) LMX_REQUIRE(seqs[j] != seqs[i], "prefill: the same sequence appears twice");
        seqs[i]->last_stream = st; seqs[i]->used = true;
        total += Ts[i];
    }
    LMX_REQUIRE(!out.hidden || n == 1, "prefill: the residual trace is for one sequence");
    if (block_rows <= 0 || block_rows > total) block_rows = (int)total;
    const int dt = cfg.dtype, gv = cfg.gemm_variant;
    Seq* s0 = seqs[0];
    constexpr int LOGIT_ROWS = 1024;                     // rows of one lm_head launch
    size_t off = 0;
    auto carve = [&](size_t bytes) { size_t o = off; off += (bytes + 255) / 256 * 256; return o; };
    int max_end = 0;                                     // longest context of this call
    for (int i = 0; i < n; ++i) max_end = std::max(max_end, seqs[i]->len + Ts[i]);
    const size_t o_h = carve(S.ids_in() ? 0 : (size_t)block_rows * H * es), o_xr = carve((size_t)block_rows * H * 4), o_x = carve((size_t)block_rows * H * es),
                 o_y = carve((size_t)block_rows * H * es), o_qkv = carve((size_t)block_rows * qkv_n * es), o_attn = carve((size_t)block_rows * S.mix_n * es),
                 o_act = carve((size_t)block_rows * I_l * es), o_log = carve((size_t)V * 4), o_want = carve((size_t)std::min(block_rows, LOGIT_ROWS) * H * es),
                 o_ws = carve(S.ws_bytes(block_rows, H, es, false)), o_scratch = carve(stack_mix_scratch(block_rows, max_end));
    if (off > s0->pws.bytes) { LMX_CHECK_HIP(hipStreamSynchronize(st)); s0->pws.ensure(off); }
    char* Wk = s0->pws.as<char>();
    void *h = Wk + o_h, *x = Wk + o_x, *y = Wk + o_y, *qkv = Wk + o_qkv, *attn = Wk + o_attn, *act = Wk + o_act, *want = Wk + o_want, *scratch = Wk + o_scratch;
    const StackWs sw = S.ws(Wk + o_ws, block_rows, H, es, false);
    float *xr = reinterpret_cast<float*>(Wk + o_xr), *last_logits = reinterpret_cast<float*>(Wk + o_log);
    if (dt != kF32 && !s0->skw.p) {
        LMX_CHECK_HIP(hipStreamSynchronize(st));
        s0->skw.ensure((size_t)256 * 256 * 256 * sizeof(float));
    }
    auto with_scratch = [&](GemmArgs g) { g.skw = s0->skw.p; return g; };
    auto rows = [&](void* base, long r0, size_t width) { return static_cast<char*>(base) + (size_t)r0 * width * es; };
    auto residual = [&](const float* xi, const void* yy, int top, const void* post, const void* inject, const void* pre, bool cast, int nr) {
        LMX_PROF("prefill.residual_norm");
        ResidualNormArgs rn{xi, yy, post, inject, pre, xr, cast ? sw.cat : x, H, S.c.width, S.c.residual_mult, S.c.norm_eps};
        rn.moe_y = sw.slots; rn.moe_w = sw.wt; rn.top = top;
        if (cast) { rn.cast = 1; rn.xn_ld = 2 * H; }
        launch_residual_norm(dt, rn, nr, st);
    };
    // what ends a sublayer: x <- x + its output, then whatever comes ahead of the next linear (`top`: experts' outputs per row to add)
    auto norm = [&](const float* xi, const void* yy, int top, const StackStep& sp, int nr) {
        if (!sp.mix) { residual(xi, yy, top, sp.post, sp.inject ? h : nullptr, sp.pre, false, nr); return; }
        residual(xi, yy, top, sp.post, nullptr, nullptr, true, nr);
        GemmArgs g{sw.cat, S.loop_in, xr, nullptr, nullptr, nr, H, 2 * H, 2 * H, 2 * H, H, 0, kActNone};
        g.c_f32 = 1;
        { LMX_PROF_K("prefill.gemm.loop"); launch_gemm(dt, g, gv, st); }
        residual(xr, nullptr, 0, nullptr, nullptr, sp.pre, false, nr);
    };
    int cur = 0, cur_done = 0;
    std::vector<int> want_next((size_t)n, 0), want_base((size_t)n, 0);      // wanted rows already served / first output row of each sequence
    for (int i = 1; i < n; ++i) want_base[(size_t)i] = want_base[(size_t)i - 1] + (out.logits ? (out.want ? (int)out.want[i - 1].size() : Ts[i - 1]) : 0);
    while (cur < n) {
        std::vector<Segment> seg;
        int fill = 0;
        while (cur < n && fill < block_rows) {
            const int take = std::min(block_rows - fill, Ts[cur] - cur_done);
            seg.push_back(Segment{cur, cur_done, fill, take, seqs[cur]->len + cur_done});
            fill += take; cur_done += take;
            if (cur_done == Ts[cur]) { ++cur; cur_done = 0; }
        }
        for (const Segment& g : seg) {
            if (S.ids_in()) {
                LMX_PROF("prefill.embed");
                EmbedRowsArgs e;
                e.ids = static_cast<const int*>(embeds[g.seq]) + g.src0;
                if (g.src0 > 0) e.prev_id = e.ids - 1; else if (g.pos0 > 0) e.prev_tok = seqs[g.seq]->d_prev;
                e.embed = embed; e.bigram = S.bigram; e.x = xr + (size_t)g.dst0 * H; e.H = H; e.vocab = Vr;
                if (S.c.loop_mix) { e.x0 = static_cast<char*>(rows(sw.cat, g.dst0, 2 * H)) + (size_t)H * es; e.x0_ld = 2 * H; }
                e.buckets = S.c.bigram_buckets; e.mul_prev = S.c.bigram_mul_prev; e.mul_cur = S.c.bigram_mul_cur;
                launch_embed_rows(dt, e, g.n, st);
                continue;
            }
            const char* src = static_cast<const char*>(embeds[g.seq]) + (size_t)g.src0 * H * es;
            LMX_CHECK_HIP(hipMemcpyAsync(rows(h, g.dst0, H), src, (size_t)g.n * H * es, hipMemcpyDeviceToDevice, st));
            if (S.c.loop_mix) LMX_CHECK_HIP(hipMemcpy2DAsync(static_cast<char*>(rows(sw.cat, g.dst0, 2 * H)) + (size_t)H * es, (size_t)2 * H * es, src, (size_t)H * es, (size_t)H * es, (size_t)g.n, hipMemcpyDeviceToDevice, st));
        }
        // x = the embedding rows
        {
            const StackRun& r0 = S.runs[0];
            const void* n1 = S.layers[(size_t)r0.layer].n1;
            if (!S.ids_in() && r0.mix) residual(nullptr, nullptr, 0, nullptr, h, nullptr, false, fill);
            norm(S.ids_in() || r0.mix ? xr : nullptr, nullptr, 0, StackStep{nullptr, n1, !S.ids_in() && !r0.mix, r0.mix}, fill);
        }
        for (int r = 0; r < L; ++r) {
            const StackLayer& l = S.layers[(size_t)S.runs[(size_t)r].layer];
            const lmx_layer_config& d = l.c;
            const int an = l.an;
            { LMX_PROF_K("prefill.gemm.qkv"); launch_gemm(dt, with_scratch(GemmArgs{x, l.wqkv, qkv, l.bqkv, nullptr, fill, l.qkv_n, H, H, H, l.qkv_n, 0, kActNone}), gv, st); }
            if (d.mixer != LMX_MIXER_ATTENTION) stack_mix_prefill(r, seqs, seg, fill, x, qkv, attn, scratch, s0->skw.p, st);
            else for (const Segment& g : seg) {
                Seq* s = seqs[g.seq];
                void *kc = s->kc.as<char>() + S.runs[(size_t)r].k_off, *vt = s->vt.as<char>() + S.runs[(size_t)r].v_off;
                void *qr = rows(qkv, g.dst0, l.qkv_n), *ar = rows(attn, g.dst0, l.out_k);
                { LMX_PROF("prefill.norm_rope_kv"); launch_qkv_norm_rope_kv(dt, l.D, rope_args(S, l, qr, kc, vt, g.n, g.pos0, s_max), st); }
                LMX_PROF("prefill.attn");
                FlashArgs fa{qr, ar, kc, vt, g.n, g.pos0 + g.n, g.pos0, l.qkv_n, l.out_k, d.n_heads, d.n_kv_heads, s_max, d.attn_scale, 1};
                fa.win = 1; fa.window = d.window; fa.sink = d.softmax_sink; fa.gate = l.gate_off >= 0 ? static_cast<char*>(qr) + (size_t)l.gate_off * es : nullptr;
                if (dt == kF32 || l.D > 128) launch_rows_attn(dt, l.D, fa, st); else launch_flash_prefill(dt, l.D, fa, st);
            }
            auto gate_up = [&](void* dst, int ld) {
                LMX_PROF_K("prefill.gemm.gate_up");
                launch_gemm(dt, with_scratch(GemmArgs{x, l.wgu, dst, nullptr, nullptr, fill, 2 * l.ff, H, H, H, ld, 0, l.act()}), gv, st);
            };
            if (l.parallel() && l.dense()) gate_up(static_cast<char*>(attn) + (size_t)an * es, l.out_k);
            { LMX_PROF_K("prefill.gemm.o"); launch_gemm(dt, with_scratch(GemmArgs{attn, l.wo, y, nullptr, nullptr, fill, H, l.out_k, l.out_k, l.out_k, H, 0, kActNone}), gv, st); }
            const void* yy = y;
            if (l.ff && !l.parallel()) {
                norm(xr, y, 0, stack_step(S, r, 0, final_norm), fill);
                if (l.dense()) {
                    gate_up(act, l.ff);
                    { LMX_PROF_K("prefill.gemm.down"); launch_gemm(dt, with_scratch(GemmArgs{act, l.wd, y, nullptr, nullptr, fill, H, l.ff, l.ff, l.ff, H, 0, kActNone}), gv, st); }
                } else yy = nullptr;
            }
            const int top = l.moe() ? d.top_experts : 0;
            if (top) stack_moe(l, x, fill, sw, stack_prof_prefill, st);
            const StackStep sp = stack_step(S, r, l.ff && !l.parallel() ? 1 : 0, final_norm);
            if (out.hidden) {
                // residual trace: the stream right after this run, before anything the next run adds
                residual(xr, yy, top, sp.post, nullptr, nullptr, false, fill);
                LMX_CHECK_HIP(hipMemcpyAsync(out.hidden + ((size_t)r * Ts[0] + seg[0].src0) * H, xr, (size_t)fill * H * 4, hipMemcpyDeviceToDevice, st));
                norm(xr, nullptr, 0, sp, fill);
            } else norm(xr, yy, top, sp, fill);
        }
        // logits of the wanted rows of this piece (x holds the finally normalised rows)
        if (out.logits)
            for (const Segment& g : seg) {
                std::vector<int> rws;                     // rows of this segment, ascending (relative to the sequence's new rows)
                if (!out.want) { rws.resize((size_t)g.n); for (int i = 0; i < g.n; ++i) rws[(size_t)i] = g.src0 + i; }
                else { const auto& w = out.want[g.seq]; int& p = want_next[(size_t)g.seq]; while (p + (int)rws.size() < (int)w.size() && w[(size_t)p + rws.size()] < g.src0 + g.n) rws.push_back(w[(size_t)p + rws.size()]); }
                for (size_t r0 = 0; r0 < rws.size(); r0 += LOGIT_ROWS) {
                    const int nr = (int)std::min(rws.size() - r0, (size_t)std::min(block_rows, LOGIT_ROWS));
                    for (int i = 0; i < nr;) {            // consecutive rows in one copy
                        int k = i + 1;
                        while (k < nr && rws[r0 + k] == rws[r0 + k - 1] + 1) ++k;
                        LMX_CHECK_HIP(hipMemcpyAsync(rows(want, i, H), rows(x, g.dst0 + rws[r0 + i] - g.src0, H), (size_t)(k - i) * H * es, hipMemcpyDeviceToDevice, st));
                        i = k;
                    }
                    GemmArgs ga{want, lm_head, out.logits + (size_t)(want_base[(size_t)g.seq] + want_next[(size_t)g.seq]) * V, nullptr, nullptr, nr, V, H, H, H, V, 0, kActNone};
                    ga.c_f32 = 1; ga.cap = S.c.logit_softcap;
                    { LMX_PROF("prefill.gemm.lm_head"); launch_gemm(dt, ga, gv, st); }
                    want_next[(size_t)g.seq] += nr;
                }
            }
        for (const Segment& g : seg) {
            if (g.src0 + g.n != Ts[g.seq] || !(greedy || out.last_logits)) continue;
            Seq* s = seqs[g.seq];
            float* dst = out.last_logits ? out.last_logits + (size_t)g.seq * V : last_logits;
            GemvArgs ga{rows(x, g.dst0 + g.n - 1, H), lm_head, dst, nullptr, nullptr, nullptr, 0.f, V, H, H, H, V, 0, kActNone};
            ga.c_f32 = 1; ga.cap = S.c.logit_softcap;
            { LMX_PROF_K("prefill.gemv.lm_head"); launch_gemv(dt, ga, 1, st); }
            if (!greedy) continue;
            if (s->samp.temperature > 0.f) launch_sample(kF32, dst, Vr, s->samp, s->d_nout, s->d_tok, nullptr, nullptr, st);
            else launch_argmax(kF32, dst, Vr, s->d_tok, st);
            launch_log_token(s->d_tok, s->d_log, s->d_nout, s->log_cap, s->d_stop, st);
        }
    }
    for (int i = 0; i < n; ++i) {
        seqs[i]->len += Ts[i];
        if (S.ids_in()) launch_set_prev(seqs[i]->d_prev, static_cast<const int*>(embeds[i]) + Ts[i] - 1, nullptr, st);
        launch_set_state(seqs[i]->d_len, seqs[i]->len, seqs[i]->d_tok, 0, 0, seqs[i]->d_nout, -1, st);
    }
}

// ---------------------------------------------------------------------------------------------------------------
// decode
// ---------------------------------------------------------------------------------------------------------------
static WinDecodeArgs decode_args(const Stack& S, const StackLayer& l, const void* qkv, void* out, int n_seq, int max_len, int s_max) {
    const lmx_layer_config& d = l.c;
    WinDecodeArgs a;
    a.qkv = qkv; a.out = out; a.q_norm = l.qn; a.k_norm = l.kn; a.cos_sin = d.rope_dims ? S.rope[(size_t)d.rope_table] : nullptr;
    a.n_seq = n_seq; a.qkv_stride = l.qkv_n; a.out_stride = l.out_k; a.n_heads = d.n_heads; a.n_kv_heads = d.n_kv_heads; a.s_max = s_max;
    a.qk_dim = d.qk_dim; a.rot_dims = d.rope_dims; a.window = d.window; a.sink = d.softmax_sink; a.gate_off = l.gate_off; a.scale = d.attn_scale; a.eps = S.c.norm_eps;
    // chunks the longest member's window can touch; enough workgroups to fill the chip, no more
    int span = max_len + 1;
    if (d.window > 0 && d.window + 127 < span) span = d.window + 127;
    const int chunks = std::max(1, std::min((span + 127) / 128, 32));
    const int fill = (1024 + d.n_heads * n_seq - 1) / (d.n_heads * n_seq);
    a.n_split = std::max(1, std::min(chunks, fill));
    return a;
}

DecodeFusedSeq Model::stack_seq_ref(int r, Seq* s) const {
    const StackRun& u = stk->runs[(size_t)r];
    const int mixer = stk->layers[(size_t)u.layer].c.mixer;
    if (mixer == LMX_MIXER_DELTA) return DecodeFusedSeq{s->rs.as<char>() + u.s_off, s->rs.as<char>() + u.r_off, s->d_len, s->d_aws, s->d_cnt, &s->d_stop->done};
    return DecodeFusedSeq{s->kc.as<char>() + u.k_off, mixer == LMX_MIXER_ATTENTION ? s->vt.as<char>() + u.v_off : nullptr, s->d_len, s->d_aws, s->d_cnt, nullptr};
}

void Model::stack_decode_step(Seq* s, hipStream_t st, int64_t* id_out) {
    Stack& S = *stk;
    const int dt = cfg.dtype;
    // the linear behind a norm: residual addition, both norms and the linear in one launch where the weight stream allows it (16-bit); the residual alternates between
    // two rows because every workgroup of that launch reads the old one
    float* xr[2] = {s->d_xr, s->d_xr + H};
    int cur = -1;                                            // row that holds x (-1: none yet, x is the embedding row)
    // norm launch in front of linears that share its row
    auto residual = [&](const StackStep& sp, const void* y, int top, bool cast) {
        LMX_PROF_K("decode.residual_norm");
        const int nxt = cur == 0 ? 1 : 0;
        ResidualNormArgs rn{cur < 0 ? nullptr : xr[cur], y, sp.post, sp.inject ? s->d_h : nullptr, cast ? nullptr : sp.pre, xr[nxt], cast ? s->sw.cat : s->d_x, H, S.c.width, S.c.residual_mult, S.c.norm_eps};
        rn.moe_y = s->sw.slots; rn.moe_w = s->sw.wt; rn.top = top;
        if (cast) { rn.cast = 1; rn.xn_ld = 2 * H; }
        cur = nxt;
        launch_residual_norm(dt, rn, 1, st);
    };
    auto plain = [&](const char* name, const void* xin, const void* w, void* c, int N, int K, int act = kActNone, bool f32 = false) {
        LMX_PROF_K(name);
        GemvArgs g{xin, w, c, nullptr, nullptr, nullptr, 0.f, N, K, K, K, act_gated(act) ? N / 2 : N, 0, act};
        g.c_f32 = f32;
        launch_gemv(dt, g, 1, st);
    };
    // a pass of the loop begins: x <- W [x; embedding row]
    auto mix_in = [&](StackStep& sp, const void*& y, int& top) {
        if (!sp.mix) return;
        residual(sp, y, top, true);
        const int nxt = cur == 0 ? 1 : 0;
        plain("decode.gemv.loop", s->sw.cat, S.loop_in, xr[nxt], H, 2 * H, kActNone, true);
        cur = nxt; y = nullptr; top = 0;
        sp = StackStep{nullptr, sp.pre, false, false};
    };
    auto linear = [&](const char* name, const StackStep& sp, const void* y, int top, GemvArgs g, bool fuse) {
        if (fuse && opt_stack_fuse && top == 0 && gemv_residual_applies(dt, g)) {
            const int nxt = cur == 0 ? 1 : 0;
            const ResidualNormArgs rn{cur < 0 ? nullptr : xr[cur], y, sp.post, sp.inject ? s->d_h : nullptr, sp.pre, xr[nxt], s->d_x, H, S.c.width, S.c.residual_mult, S.c.norm_eps};
            cur = nxt;
            LMX_PROF_K(name);
            launch_gemv_residual(dt, g, rn, st);
            return;
        }
        residual(sp, y, top, false);
        LMX_PROF_K(name);
        g.X = s->d_x;
        launch_gemv(dt, g, 1, st);
    };
    StackStep before{nullptr, S.layers[(size_t)S.runs[0].layer].n1, !S.ids_in(), S.runs[0].mix};
    const void* y = nullptr;
    int top = 0;                                             // experts' outputs waiting to be added
    if (S.ids_in()) {
        LMX_PROF_K("decode.embed");
        EmbedRowsArgs e;
        e.tok = s->d_tok; e.prev_tok = s->d_prev;
        e.embed = embed; e.bigram = S.bigram; e.x = xr[0]; e.H = H; e.vocab = Vr;
        if (S.c.loop_mix) { e.x0 = static_cast<char*>(s->sw.cat) + (size_t)H * es; e.x0_ld = 2 * H; }
        e.buckets = S.c.bigram_buckets; e.mul_prev = S.c.bigram_mul_prev; e.mul_cur = S.c.bigram_mul_cur;
        launch_embed_rows(dt, e, 1, st);
        cur = 0;
    } else if (S.c.loop_mix) LMX_CHECK_HIP(hipMemcpyAsync(static_cast<char*>(s->sw.cat) + (size_t)H * es, s->d_h, (size_t)H * es, hipMemcpyDeviceToDevice, st));
    for (int r = 0; r < L; ++r) {
        const StackLayer& l = S.layers[(size_t)S.runs[(size_t)r].layer];
        mix_in(before, y, top);
        const GemvArgs g{nullptr, l.wqkv, s->d_qkv, l.bqkv, nullptr, nullptr, 0.f, l.qkv_n, H, H, H, l.qkv_n, 0, kActNone};
        linear("decode.gemv.qkv", before, y, top, g, !(l.parallel() && l.ff));      // a parallel layer's other linears read the same row
        top = 0;
        if (l.c.mixer == LMX_MIXER_ATTENTION) {
            LMX_PROF_K("decode.attn");
            WinDecodeArgs a = decode_args(S, l, s->d_qkv, s->d_attn, 1, s->len, s_max);
            a.one = stack_seq_ref(r, s);
            a.pos = s->len;
            launch_decode_win(dt, l.D, a, st);
        } else stack_mix_decode(r, nullptr, stack_seq_ref(r, s), 1, s->len, s->d_qkv, s->d_attn, s->sw, nullptr, st);
        if (l.parallel() && l.dense()) plain("decode.gemv.gate_up", s->d_x, l.wgu, static_cast<char*>(s->d_attn) + (size_t)l.an * es, 2 * l.ff, H, l.act());
        plain("decode.gemv.o", s->d_attn, l.wo, s->d_y, H, l.out_k);
        y = s->d_y;
        if (l.ff && !l.parallel()) {
            const StackStep sp = stack_step(S, r, 0, final_norm);
            if (l.dense()) {
                linear("decode.gemv.gate_up", sp, y, 0, GemvArgs{nullptr, l.wgu, s->d_act, nullptr, nullptr, nullptr, 0.f, 2 * l.ff, H, H, H, l.ff, 0, l.act()}, true);
                plain("decode.gemv.down", s->d_act, l.wd, s->d_y, H, l.ff);
            } else { residual(sp, y, 0, false); y = nullptr; }
        }
        if (l.moe()) { stack_moe(l, s->d_x, 1, s->sw, stack_prof_decode, st); top = l.c.top_experts; }
        before = stack_step(S, r, l.ff && !l.parallel() ? 1 : 0, final_norm);
    }
    {
        GemvArgs ga{nullptr, lm_head, s->d_logits, nullptr, nullptr, nullptr, 0.f, V, H, H, H, V, 0, kActNone};
        ga.c_f32 = 1; ga.cap = S.c.logit_softcap;
        linear("decode.gemv.lm_head", before, y, top, ga, false);      // one row of residual_norm is cheaper than forming it in every workgroup of a vocabulary-wide linear
    }
    LMX_PROF("decode.argmax");
    const SeqStateRef ref{s->d_len, s->d_nout, s->d_tok, s->d_log, s->log_cap, 0, s->samp, s->d_stop, S.ids_in() ? s->d_prev : nullptr};
    launch_argmax_advance_batch(dt, s->d_logits, Vr, V, nullptr, &ref, 1, id_out, S.ids_in() ? nullptr : embed, s->d_h, H, st, /*f32_logits=*/true);
}

void Model::stack_decode_batch_step(Batch* b, Seq* const* seqs, int n, int64_t* ids, hipStream_t st) {
    Stack& S = *stk;
    const int dt = cfg.dtype;
    auto residual = [&](const float* xi, const void* yy, int top, const void* post, const void* inject, const void* pre, bool cast) {
        LMX_PROF("decode_batch.residual_norm");
        ResidualNormArgs rn{xi, yy, post, inject, pre, b->xr, cast ? b->sw.cat : b->x, H, S.c.width, S.c.residual_mult, S.c.norm_eps};
        rn.moe_y = b->sw.slots; rn.moe_w = b->sw.wt; rn.top = top;
        if (cast) { rn.cast = 1; rn.xn_ld = 2 * H; }
        launch_residual_norm(dt, rn, n, st);
    };
    auto linear = [&](GemmArgs g, const void* wsw) { LMX_PROF("decode_batch.linear"); stack_batch_linear(b, g, wsw, st); };
    auto norm = [&](const float* xi, const void* yy, int top, const StackStep& sp) {
        if (!sp.mix) { residual(xi, yy, top, sp.post, sp.inject ? b->h : nullptr, sp.pre, false); return; }
        residual(xi, yy, top, sp.post, nullptr, nullptr, true);
        GemmArgs g{b->sw.cat, S.loop_in, b->xr, nullptr, nullptr, n, H, 2 * H, 2 * H, 2 * H, H, 0, kActNone};
        g.c_f32 = 1;
        linear(g, S.sw_loop);
        residual(b->xr, nullptr, 0, nullptr, nullptr, sp.pre, false);
    };
    int max_len = 0;
    for (int i = 0; i < n; ++i) max_len = std::max(max_len, seqs[i]->len);
    const StackRun& r0 = S.runs[0];
    if (S.ids_in()) {
        LMX_PROF("decode_batch.embed");
        EmbedRowsArgs e;
        e.tab = b->d_state_tab;
        e.embed = embed; e.bigram = S.bigram; e.x = b->xr; e.H = H; e.vocab = Vr;
        if (S.c.loop_mix) { e.x0 = static_cast<char*>(b->sw.cat) + (size_t)H * es; e.x0_ld = 2 * H; }
        e.buckets = S.c.bigram_buckets; e.mul_prev = S.c.bigram_mul_prev; e.mul_cur = S.c.bigram_mul_cur;
        launch_embed_rows(dt, e, n, st);
    } else if (S.c.loop_mix) {
        LMX_CHECK_HIP(hipMemcpy2DAsync(static_cast<char*>(b->sw.cat) + (size_t)H * es, (size_t)2 * H * es, b->h, (size_t)H * es, (size_t)H * es, (size_t)n, hipMemcpyDeviceToDevice, st));
        if (r0.mix) residual(nullptr, nullptr, 0, nullptr, b->h, nullptr, false);
    }
    norm(S.ids_in() || r0.mix ? b->xr : nullptr, nullptr, 0, StackStep{nullptr, S.layers[(size_t)r0.layer].n1, !S.ids_in() && !r0.mix, r0.mix});
    for (int r = 0; r < L; ++r) {
        const StackLayer& l = S.layers[(size_t)S.runs[(size_t)r].layer];
        linear(GemmArgs{b->x, l.wqkv, b->qkv, l.bqkv, nullptr, n, l.qkv_n, H, H, H, l.qkv_n, 0, kActNone}, l.sw_qkv);
        const DecodeFusedSeq* tab = b->d_attn_tab + (size_t)r * b->cap;
        if (l.c.mixer == LMX_MIXER_ATTENTION) {
            LMX_PROF("decode_batch.attn");
            WinDecodeArgs a = decode_args(S, l, b->qkv, b->attn, n, max_len, s_max);
            a.tab = tab;
            launch_decode_win(dt, l.D, a, st);
        } else stack_mix_decode(r, tab, DecodeFusedSeq{}, n, max_len, b->qkv, b->attn, b->sw, b, st);
        if (l.parallel() && l.dense()) linear(GemmArgs{b->x, l.wgu, static_cast<char*>(b->attn) + (size_t)l.an * es, nullptr, nullptr, n, 2 * l.ff, H, H, H, l.out_k, 0, l.act()}, l.sw_gu);
        linear(GemmArgs{b->attn, l.wo, b->y, nullptr, nullptr, n, H, l.out_k, l.out_k, l.out_k, H, 0, kActNone}, l.sw_o);
        const void* yy = b->y;
        if (l.ff && !l.parallel()) {
            norm(b->xr, b->y, 0, stack_step(S, r, 0, final_norm));
            if (l.dense()) {
                linear(GemmArgs{b->x, l.wgu, b->act, nullptr, nullptr, n, 2 * l.ff, H, H, H, l.ff, 0, l.act()}, l.sw_gu);
                linear(GemmArgs{b->act, l.wd, b->y, nullptr, nullptr, n, H, l.ff, l.ff, l.ff, H, 0, kActNone}, l.sw_d);
            } else yy = nullptr;
        }
        if (l.moe()) stack_moe(l, b->x, n, b->sw, stack_prof_batch, st);
        norm(b->xr, yy, l.moe() ? l.c.top_experts : 0, stack_step(S, r, l.ff && !l.parallel() ? 1 : 0, final_norm));
    }
    GemmArgs ga{b->x, lm_head, b->logits, nullptr, nullptr, n, V, H, H, H, V, 0, kActNone};
    ga.c_f32 = 1; ga.cap = S.c.logit_softcap;
    linear(ga, sw_lm_head);
    LMX_PROF("decode_batch.argmax");
    launch_argmax_advance_batch(dt, b->logits, Vr, V, b->d_state_tab, nullptr, n, ids, S.ids_in() ? nullptr : embed, b->h, H, st, /*f32_logits=*/true);
}

void Model::stack_batch_linear(Batch* b, GemmArgs g, const void* wsw, hipStream_t st) {
    if (cfg.dtype != kF32 && g.M <= 32) {
        g.Wsw = wsw;
        if (!g.c_f32) { g.skw = b->sk_scratch.p; g.sk_cnt = b->sk_cnt.as<int>(); }
        launch_skinny_gemm(cfg.dtype, g, st);
    } else launch_gemm(cfg.dtype, g, cfg.gemm_variant, st);
}

void Model::stack_seq_copy(Seq* dst, const Seq* src, hipStream_t st) {
    const size_t n = (size_t)src->len;
    for (const StackRun& r : stk->runs) {
        const StackLayer& l = stk->layers[(size_t)r.layer];
        const size_t nk = (size_t)l.c.n_kv_heads;
        if (l.c.mixer == LMX_MIXER_LATENT) LMX_CHECK_HIP(hipMemcpyAsync(dst->kc.as<char>() + r.k_off, src->kc.as<char>() + r.k_off, n * l.R * es, hipMemcpyDeviceToDevice, st));
        if (l.c.mixer != LMX_MIXER_ATTENTION) continue;
        LMX_CHECK_HIP(hipMemcpy2DAsync(dst->kc.as<char>() + r.k_off, (size_t)s_max * l.D * es, src->kc.as<char>() + r.k_off, (size_t)s_max * l.D * es, n * l.D * es, nk, hipMemcpyDeviceToDevice, st));
        LMX_CHECK_HIP(hipMemcpy2DAsync(dst->vt.as<char>() + r.v_off, (size_t)s_max * es, src->vt.as<char>() + r.v_off, (size_t)s_max * es, n * es, nk * l.D, hipMemcpyDeviceToDevice, st));
    }
    if (stk->s_bytes) LMX_CHECK_HIP(hipMemcpyAsync(dst->rs.p, src->rs.p, stk->s_bytes, hipMemcpyDeviceToDevice, st));
    if (stk->ids_in()) launch_set_prev(dst->d_prev, nullptr, src->d_prev, st);
}

}  // namespace lmx
