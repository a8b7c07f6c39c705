// Mixers and mixtures of the layer-stack decoders besides softmax attention (stack.cpp): launch sequences of latent attention, the gated delta rule and the mixture of
// experts, for the rows of a prompt piece and for one new token per sequence.
#include "engine.h"

namespace lmx {

struct StackProf { const char *delta, *norm, *uq, *qlat, *attn, *olat, *router, *plan, *gate_up, *down; };
#define NAMES(P, UQ) {P ".delta", P ".latent_norm", UQ, P ".latent_q", P ".attn", P ".latent_o", P ".moe.router", P ".moe.plan", P ".moe.gate_up", P ".moe.down"}
const StackProf stack_prof_prefill = NAMES("prefill", "prefill.gemm.uq"), stack_prof_decode = NAMES("decode", "decode.gemv.uq"), stack_prof_batch = NAMES("decode_batch", "decode_batch.linear");
#undef NAMES

static int round_up(int a, int b) { return (a + b - 1) / b * b; }
static size_t up256(size_t b) { return (b + 255) / 256 * 256; }

size_t Stack::ws_bytes(int rows, int H, int es, bool decode) const {
    const size_t r = (size_t)rows;
    return (decode ? up256(r * q_n * es) + 2 * up256(r * lat_n * es) : 0) + up256(r * moe_act * es) + up256(r * moe_top * H * es) + 2 * up256(r * moe_top * 4) +
           (moe_top ? up256(group_plan_bytes(rows * moe_top)) : 0) + (c.loop_mix ? up256(r * 2 * H * es) : 0);
}

StackWs Stack::ws(void* base, int rows, int H, int es, bool decode) const {
    char* p = static_cast<char*>(base);
    const size_t r = (size_t)rows;
    auto take = [&](size_t bytes) -> void* { void* q = p; p += up256(bytes); return q; };
    StackWs w{};
    if (decode) { w.q = take(r * q_n * es); w.qlat = take(r * lat_n * es); w.olat = take(r * lat_n * es); }
    w.act = take(r * moe_act * es);
    w.slots = take(r * moe_top * H * es);
    w.ids = static_cast<int*>(take(r * moe_top * 4));
    w.wt = static_cast<float*>(take(r * moe_top * 4));
    if (moe_top) w.plan = take(group_plan_bytes(rows * moe_top));
    if (c.loop_mix) w.cat = take(r * 2 * H * es);
    return w;
}

// ---------------------------------------------------------------------------------------------------------------
// prompt rows
// ---------------------------------------------------------------------------------------------------------------
// keys [k0, end) that the rows of a segment can see, k0 on a 64-key boundary
static int first_key(const lmx_layer_config& d, int pos0) { return d.window > 0 && pos0 - d.window + 1 > 0 ? (pos0 - d.window + 1) & ~63 : 0; }

// scratch of the widest mixer; keys: longest context of the call
size_t Model::stack_mix_scratch(int rows, int keys) const {
    size_t most = 0;
    for (const StackLayer& l : stk->layers) {
        size_t b = 0;
        if (l.c.mixer == LMX_MIXER_LATENT) {
            const int nk = l.c.window > 0 ? std::min(keys, rows + l.c.window + 64) : keys;
            b = up256((size_t)rows * l.an * es) + up256((size_t)nk * 2 * l.an * es) + 2 * up256((size_t)round_up(nk, 128) * l.an * es);
        } else if (l.c.mixer == LMX_MIXER_DELTA) b = up256((size_t)rows * l.ds.H * (l.ds.DK + l.ds.DV) * es) + delta_scratch_bytes(l.ds, rows, es);
        most = std::max(most, b);
    }
    return most;
}

void Model::stack_mix_prefill(int r, Seq* const* seqs, const std::vector<Segment>& seg, int fill, const void* x, void* qkv, void* mix, void* scratch, void* skw, hipStream_t st) {
    Stack& S = *stk;
    const StackRun& run = S.runs[(size_t)r];
    const StackLayer& l = S.layers[(size_t)run.layer];
    const lmx_layer_config& d = l.c;
    const int dt = cfg.dtype, gv = cfg.gemm_variant;
    char* p = static_cast<char*>(scratch);
    auto take = [&](size_t bytes) -> char* { char* q = p; p += up256(bytes); return q; };
    auto gemm = [&](const char* name, GemmArgs g) { LMX_PROF_K(name);
        // inner sizes of a few K-steps: the time is the launch's fixed part and the output; the smaller tiles write it sooner than the large ones
        const int v = gv == 0 && dt != kF32 && g.K <= 512 ? (g.K <= 256 ? 5 : 18) : gv;
        g.skw = g.K >= 1024 ? skw : nullptr;
        launch_gemm(dt, g, v, st); };
    if (d.mixer == LMX_MIXER_DELTA) {
        DeltaPrefillArgs a{};
        a.s = l.ds; a.w = DeltaWeights{l.conv, l.a_log, l.dt_bias, l.onorm};
        a.proj = qkv; a.ld = l.qkv_n;
        const int agn = l.ds.H * (l.ds.DK + l.ds.DV), k = l.ra + l.rg;
        void* ag = take((size_t)fill * agn * es);
        gemm("prefill.gemm.decay_gate", GemmArgs{static_cast<char*>(qkv) + (size_t)l.a_off() * es, l.wag, ag, nullptr, nullptr, fill, agn, k, l.qkv_n, k, agn, 0, kActNone});
        a.ag = ag; a.ag_ld = agn;
        delta_carve(a, p, fill, es);
        a.out = mix; a.out_ld = l.out_k; a.eps = S.c.norm_eps;
        for (size_t s0 = 0; s0 < seg.size(); s0 += DELTA_MAX_SEG) {
            a.n_seg = (int)std::min(seg.size() - s0, (size_t)DELTA_MAX_SEG);
            for (int i = 0, chunks = 0; i < a.n_seg; ++i) {
                const Segment& g = seg[s0 + (size_t)i];
                char* rs = seqs[g.seq]->rs.as<char>();
                a.seg[i] = DeltaSeg{g.dst0, g.n, g.pos0, chunks, reinterpret_cast<float*>(rs + run.s_off), rs + run.r_off};
                chunks += (g.n + 15) / 16;
            }
            { LMX_PROF_K("prefill.delta.prep"); launch_delta_prep(dt, a, st); }
            { LMX_PROF_K("prefill.delta.scan"); launch_delta_scan(dt, a, st); }
            { LMX_PROF_K("prefill.delta.gate"); launch_delta_gate(dt, a, st); }
        }
        return;
    }
    // latent attention: latents into the cache, queries, then per segment the keys and values its rows can see
    for (const Segment& g : seg) {
        LMX_PROF("prefill.latent_norm");
        LatentNormArgs n{static_cast<char*>(qkv) + (size_t)g.dst0 * l.qkv_n * es, l.qkv_n, l.Q, d.q_rank, l.R, d.kv_rank, l.qn_lat, l.kn_lat, seqs[g.seq]->kc.as<char>() + run.k_off, g.pos0};
        n.s_max = s_max; n.eps = S.c.norm_eps;
        launch_latent_norm(dt, n, g.n, st);
    }
    void* q = take((size_t)fill * l.an * es);
    gemm("prefill.gemm.uq", GemmArgs{qkv, l.wuq, q, nullptr, nullptr, fill, l.an, l.Q, l.qkv_n, l.Q, l.an, 0, kActNone});
    char* const base = p;
    for (const Segment& g : seg) {
        p = base;
        const int k0 = first_key(d, g.pos0), nk = g.pos0 + g.n - k0, cap = round_up(nk, 128);
        const char* lat = seqs[g.seq]->kc.as<char>() + run.k_off + (size_t)k0 * l.R * es;
        void* kv = take((size_t)nk * 2 * l.an * es);
        void *kc = take((size_t)cap * l.an * es), *vt = take((size_t)cap * l.an * es);
        gemm("prefill.gemm.ukv", GemmArgs{lat, l.wukv, kv, nullptr, nullptr, nk, 2 * l.an, l.R, l.R, l.R, 2 * l.an, 0, kActNone});
        {
            LMX_PROF("prefill.kv_rows");
            QkvNormRopeArgs ra{kv, kc, vt, nullptr, nullptr, nullptr, nk, 0, 2 * l.an, 0, d.n_heads, cap, l.D, 0, S.c.norm_eps};
            ra.zero_to = cap;                                // the attention tiles are whole: what lies behind the last key must not be NaN bits
            launch_qkv_norm_rope_kv(dt, l.D, ra, st);
        }
        LMX_PROF("prefill.attn");
        FlashArgs fa{static_cast<char*>(q) + (size_t)g.dst0 * l.an * es, static_cast<char*>(mix) + (size_t)g.dst0 * l.out_k * es, kc, vt, g.n, nk, g.pos0 - k0, l.an, l.out_k, d.n_heads, d.n_heads, cap,
                     d.attn_scale, 1};
        fa.win = 1; fa.window = d.window; fa.sink = d.softmax_sink;
        if (dt == kF32 || l.D > 128) launch_rows_attn(dt, l.D, fa, st); else launch_flash_prefill(dt, l.D, fa, st);
    }
}

// ---------------------------------------------------------------------------------------------------------------
// one new token per sequence
// ---------------------------------------------------------------------------------------------------------------
void Model::stack_mix_decode(int r, const DecodeFusedSeq* tab, const DecodeFusedSeq& one, int n, int max_len, void* qkv, void* mix, const StackWs& w, Batch* b, hipStream_t st) {
    Stack& S = *stk;
    const StackLayer& l = S.layers[(size_t)S.runs[(size_t)r].layer];
    const lmx_layer_config& d = l.c;
    const int dt = cfg.dtype;
    const StackProf& pn = b ? stack_prof_batch : stack_prof_decode;
    if (d.mixer == LMX_MIXER_DELTA) {
        DeltaDecodeArgs a{};
        a.s = l.ds; a.w = DeltaWeights{l.conv, l.a_log, l.dt_bias, l.onorm};
        a.proj = qkv; a.ld = l.qkv_n; a.a_off = l.a_off(); a.ra = l.ra; a.rg = l.rg;
        a.wag = l.wag; a.wag_ld = l.ra + l.rg; a.out = mix; a.out_ld = l.out_k;
        a.tab = tab; a.one = one; a.n_seq = n; a.eps = S.c.norm_eps;
        LMX_PROF_K(pn.delta);
        launch_delta_decode(dt, a, st);
        return;
    }
    {
        LMX_PROF_K(pn.norm);
        LatentNormArgs a{qkv, l.qkv_n, l.Q, d.q_rank, l.R, d.kv_rank, l.qn_lat, l.kn_lat, one.K, 0};
        a.tab = tab; a.pos_ptr = tab ? nullptr : one.pos_ptr; a.s_max = s_max; a.eps = S.c.norm_eps;
        launch_latent_norm(dt, a, n, st);
    }
    {
        LMX_PROF_K(pn.uq);
        if (b) stack_batch_linear(b, GemmArgs{qkv, l.wuq, w.q, nullptr, nullptr, n, l.an, l.Q, l.qkv_n, l.Q, l.an, 0, kActNone}, l.sw_uq, st);
        else launch_gemv(dt, GemvArgs{qkv, l.wuq, w.q, nullptr, nullptr, nullptr, 0.f, l.an, l.Q, l.qkv_n, l.Q, l.an, 0, kActNone}, 1, st);
    }
    // q W_uk of every head: the scores against all cached latents are then plain dot products
    GroupGemvArgs g{w.q, l.wuk_t, w.qlat, l.R, l.D, l.an, l.D, d.n_heads * l.R, (size_t)l.R * l.D};
    g.groups = d.n_heads; g.x_group = l.D; g.c_group = l.R;
    { LMX_PROF_K(pn.qlat); stack_heads(g, n, st); }
    {
        LMX_PROF_K(pn.attn);
        LatentDecodeArgs a;
        a.q = w.qlat; a.out = w.olat; a.tab = tab; a.one = one; a.n_seq = n; a.H = d.n_heads; a.R = l.R; a.s_max = s_max; a.window = d.window; a.scale = d.attn_scale;
        int span = max_len + 1;
        if (d.window > 0 && d.window < span) span = d.window;
        a.n_split = latent_decode_split(dt, l.R, d.n_heads, n, span);
        launch_latent_decode(dt, a, st);
    }
    GroupGemvArgs o{w.olat, static_cast<char*>(l.wukv) + (size_t)l.an * l.R * es, mix, l.D, l.R, d.n_heads * l.R, l.R, l.out_k, (size_t)l.D * l.R};
    o.groups = d.n_heads; o.x_group = l.R; o.c_group = l.D;
    { LMX_PROF_K(pn.olat); stack_heads(o, n, st); }
}

// every head's rows through the head's own weight
void Model::stack_heads(const GroupGemvArgs& g, int n, hipStream_t st) {
    const int dt = cfg.dtype;
    if (dt == kF32 || n < 4) { launch_group_gemv(dt, g, n * g.groups, st); return; }
    GroupGemmArgs a{g.X, g.W, g.C, g.N, g.K, g.ldx, g.ldw, g.ldc, g.w_group, n, g.groups};
    a.x_group = g.x_group; a.c_group = g.c_group;
    launch_group_gemm(dt, a, n <= 32 ? 32 : 64, st);
}

// ---------------------------------------------------------------------------------------------------------------
// mixture of experts: choices, then both products with the rows as they are (few: weights streamed per row) or sorted by expert (MFMA tiles)
// ---------------------------------------------------------------------------------------------------------------
void Model::stack_moe(const StackLayer& l, const void* x, int rows, const StackWs& w, const StackProf& pn, hipStream_t st) {
    const int dt = cfg.dtype, top = l.c.top_experts, E = l.c.experts, slots = rows * top;
    { LMX_PROF_K(pn.router); launch_moe_router(dt, MoeRouterArgs{x, l.wr, l.br, H, H, E, top, w.ids, w.wt}, rows, st); }
    if (group_gemm_applies(dt, slots, E)) {
        const int bm = group_gemm_bm(slots, E);
        const GroupPlan plan = group_plan_at(w.plan, slots);
        { LMX_PROF_K(pn.plan); launch_group_plan(w.ids, slots, E, bm, plan, st); }
        GroupGemmArgs g{x, l.wgu, w.act, 2 * l.ff, H, H, H, l.ff, (size_t)2 * l.ff * H, slots, E};
        g.act = l.act(); g.per_row = top; g.plan = plan;
        { LMX_PROF_K(pn.gate_up); launch_group_gemm(dt, g, bm, st); }
        GroupGemmArgs o{w.act, l.wd, w.slots, H, l.ff, l.ff, l.ff, H, (size_t)H * l.ff, slots, E};
        o.plan = plan;
        { LMX_PROF_K(pn.down); launch_group_gemm(dt, o, bm, st); }
        return;
    }
    GroupGemvArgs g{x, l.wgu, w.act, 2 * l.ff, H, H, H, l.ff, (size_t)2 * l.ff * H};
    g.act = l.act(); g.ids = w.ids; g.per_row = top;
    { LMX_PROF_K(pn.gate_up); launch_group_gemv(dt, g, slots, st); }
    GroupGemvArgs o{w.act, l.wd, w.slots, H, l.ff, l.ff, l.ff, H, (size_t)H * l.ff};
    o.ids = w.ids;
    { LMX_PROF_K(pn.down); launch_group_gemv(dt, o, slots, st); }
}

}  // namespace lmx
