// Kernels of the layer-stack decoders (stack.cpp): models described layer by layer, with an fp32 residual stream, norms on both sides of a sublayer, per-head
// query / key norms, partial rotary positions, sliding windows, a softmax sink and output gates.  Every size and constant is an argument.
//
//   residual_norm_kernel       x <- x + m rms_norm(y) w_post (+ injected row), xn <- rms_norm(x) w_pre : one launch between any two linears of a prefill / batch
//   qkv_norm_rope_kv_kernel    query / key norm, rotation, KV append of a prompt portion (q stays in its row, k rows and V^T columns go to the caches)
//   rows_attn_kernel           any dtype, VALU: one workgroup per (row, head); the fp32 engine's prefill and head widths past the MFMA kernel's
//   decode_win_kernel          one new token per sequence: query / key norm, rotation, append, attention over the window, sink, gate, split merge in one launch
// (16-bit prefill attention with head widths up to 128 is flash_prefill2_kernel's windowed form, attention.hip.)
//
// Head vectors are stored padded to D in {64, 128, 256} lanes: the padding weights are zero, so padded lanes of q, k and v are zero and add nothing; the query / key
// norm divides by the true width.
#include "common.h"
#include "kernels.h"
#include "attention_decode.h"

namespace lmx {

// ---------------------------------------------------------------------------------------------------------------
// residual + norms
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int NP>
__global__ __launch_bounds__(256) void residual_norm_kernel(ResidualNormArgs a) {
    __shared__ float red[4];
    const int row = blockIdx.x, tid = threadIdx.x, HC = a.H >> 3;
    const float rH = 1.f / (float)a.H_real;
    const float* xin = a.x_in ? a.x_in + (size_t)row * a.H : nullptr;
    const T* y = a.y ? reinterpret_cast<const T*>(a.y) + (size_t)row * a.H : nullptr;
    const T* inj = a.inject ? reinterpret_cast<const T*>(a.inject) + (size_t)row * a.H : nullptr;
    const T* post = y || a.top > 0 ? reinterpret_cast<const T*>(a.post_w) : nullptr;
    const T* pre = reinterpret_cast<const T*>(a.pre_w);
    float x[NP][8], yv[NP][8];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
        const int c = tid + i * 256;
        if (c >= HC) continue;
        if (xin) load8<float>(xin + c * 8, x[i]);
        else {
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] = 0.f;
        }
        if (y) load8<T>(y + c * 8, yv[i]);
        else {
#pragma unroll
            for (int e = 0; e < 8; ++e) yv[i][e] = 0.f;
        }
        for (int k = 0; k < a.top; ++k) {
            const float wk = a.moe_w[(size_t)row * a.top + k];
            float v[8]; load8<T>(reinterpret_cast<const T*>(a.moe_y) + ((size_t)row * a.top + k) * a.H + c * 8, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) yv[i][e] = fmaf(wk, v[e], yv[i][e]);
        }
        if (post) {
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += yv[i][e] * yv[i][e];
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] += a.mult * yv[i][e];
        }
    }
    if (post) {
        ss = block_sum<4>(ss, red);
        const float inv = a.mult / sqrtf(ss * rH + a.eps);
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int c = tid + i * 256;
            if (c >= HC) continue;
            float g[8]; load8<T>(post + c * 8, g);
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] += yv[i][e] * inv * g[e];
        }
    }
    float s2 = 0.f;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
        const int c = tid + i * 256;
        if (c >= HC) continue;
        if (inj) {
            float g[8]; load8<T>(inj + c * 8, g);
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] += g[e];
        }
        if (a.x_out) store8<float>(a.x_out + (size_t)row * a.H + c * 8, x[i]);
#pragma unroll
        for (int e = 0; e < 8; ++e) s2 += x[i][e] * x[i][e];
    }
    T* xn = reinterpret_cast<T*>(a.xn) + (size_t)row * (a.xn_ld ? a.xn_ld : a.H);
    if (a.cast) {
#pragma unroll
        for (int i = 0; i < NP; ++i) { const int c = tid + i * 256; if (c < HC) store8<T>(xn + c * 8, x[i]); }
        return;
    }
    if (!pre) return;
    s2 = block_sum<4>(s2, red);
    const float inv2 = 1.f / sqrtf(s2 * rH + a.eps);
#pragma unroll
    for (int i = 0; i < NP; ++i) {
        const int c = tid + i * 256;
        if (c >= HC) continue;
        float g[8], o[8]; load8<T>(pre + c * 8, g);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = x[i][e] * inv2 * g[e];
        store8<T>(xn + c * 8, o);
    }
}

// ---------------------------------------------------------------------------------------------------------------
// input rows of a model whose embedding depends on the token before: x = embed[t] + bigram[(prev mul_prev + t mul_cur) mod buckets] (row `buckets` without a previous
// token), summed in fp32.  One workgroup per row.
// ---------------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(EmbedRowsArgs a) {
    const int row = blockIdx.x, tid = threadIdx.x;
    int64_t t, prev = -1;
    if (a.tab) { t = *a.tab[row].tok; prev = *a.tab[row].prev; }
    else if (a.ids) {
        t = a.ids[row];
        if (row > 0) prev = a.ids[row - 1];
        else if (a.prev_id) prev = *a.prev_id;
        else if (a.prev_tok) prev = *a.prev_tok;
    } else { t = *a.tok; prev = *a.prev_tok; }
    t = t < 0 ? 0 : (t >= a.vocab ? a.vocab - 1 : t);
    int64_t b = a.buckets;
    if (prev >= 0) {
        b = (prev * a.mul_prev + t * a.mul_cur) % a.buckets;
        if (b < 0) b += a.buckets;
    }
    const T* e = reinterpret_cast<const T*>(a.embed) + (size_t)t * a.H;
    const T* g = reinterpret_cast<const T*>(a.bigram) + (size_t)b * a.H;
    for (int c = tid; c < (a.H >> 3); c += 256) {
        float v[8], u[8];
        load8<T>(e + c * 8, v); load8<T>(g + c * 8, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] += u[i];
        store8<float>(a.x + (size_t)row * a.H + c * 8, v);
        if (a.x0) store8<T>(reinterpret_cast<T*>(a.x0) + (size_t)row * a.x0_ld + c * 8, v);
    }
}

void launch_embed_rows(int dtype, const EmbedRowsArgs& a, int rows, hipStream_t st) {
    LMX_REQUIRE(a.embed && a.bigram && a.x && a.buckets >= 1 && a.H % 8 == 0 && a.vocab >= 1, "embed_rows: bad arguments");
    LMX_REQUIRE(a.tab || a.ids || (rows == 1 && a.tok && a.prev_tok), "embed_rows: no tokens");
    LMX_REQUIRE(!a.x0 || a.x0_ld % 8 == 0, "embed_rows: bad pitch");
    if (rows <= 0) return;
#define L(TT) LMX_LAUNCH(embed_rows_kernel<TT>, dim3(rows), dim3(256), 0, st, a)
    if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

void launch_residual_norm(int dtype, const ResidualNormArgs& a, int rows, hipStream_t st) {
    LMX_REQUIRE(a.H % 8 == 0 && a.H > 0 && a.H <= 8192 && a.H_real >= 1 && a.H_real <= a.H, "residual_norm: width must be a multiple of 8, at most 8192");
    LMX_REQUIRE(a.top >= 0 && (a.top == 0 || (a.moe_y && a.moe_w)), "residual_norm: expert outputs need their weights");
    LMX_REQUIRE((!a.pre_w && !a.cast) || a.xn, "residual_norm: the normalised rows need a buffer");
    LMX_REQUIRE(!(a.pre_w && a.cast) && a.xn_ld % 8 == 0, "residual_norm: norm or cast, in 16-byte rows");
    if (rows <= 0) return;
    const int np = (a.H / 8 + 255) / 256;
#define R(TT, NPV) LMX_LAUNCH((residual_norm_kernel<TT, NPV>), dim3(rows), dim3(256), 0, st, a)
#define RT(TT) do { if (np == 1) R(TT, 1); else if (np == 2) R(TT, 2); else R(TT, 4); } while (0)
    if (dtype == kBF16) RT(bf16_t); else if (dtype == kF16) RT(f16_t); else RT(float);
#undef RT
#undef R
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// query / key norm + rotation + KV append of prompt rows.  grid (ceil(T / 64), H + 2 G), 256 threads.
//   PAIRED (rot_dims % 16 == 0): D / 16 lanes own one head vector, two 8-element chunks each — a chunk of the rotated part with its partner half a rotation away, or two
//   neighbouring chunks of the rest — so a lane rotates what it loaded: no LDS, no barrier.
//   otherwise: D / 8 lanes, 8 consecutive elements each, the partner i +- rot_dims / 2 through LDS (any even number of rotated dimensions).
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int D, bool PAIRED>
__global__ __launch_bounds__(256) void qkv_norm_rope_kv_kernel(QkvNormRopeArgs a) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x;
    const int tok0 = blockIdx.x * 64, slot = blockIdx.y;
    const int ntok = (a.T - tok0) < 64 ? (a.T - tok0) : 64;                // <= 0: a block of nothing but rows to clear
    const int nzero = (a.zero_to - tok0) < 64 ? (a.zero_to - tok0) : 64;
    T* qkv = reinterpret_cast<T*>(a.qkv);
    constexpr int LPV = D / 8, VPP = 256 / LPV;          // lanes per vector, vectors per pass
    if (PAIRED && slot < a.n_heads + a.n_kv_heads) {
        constexpr int LP = D / 16, ITER = 64 * LP / 256;
        const bool is_k = slot >= a.n_heads;
        const int half8 = a.rot_dims >> 4, k = tid % LP;                   // rotated chunks per half
        const bool rot = k < half8;
        const int c0 = rot ? k : 2 * half8 + 2 * (k - half8), c1 = rot ? k + half8 : c0 + 1;
        const T* nw = reinterpret_cast<const T*>(is_k ? a.k_norm : a.q_norm);
        T* kc = reinterpret_cast<T*>(a.K) + (size_t)(is_k ? slot - a.n_heads : 0) * a.s_max * D;
        float x[ITER][2][8], g0[8], g1[8];
#pragma unroll
        for (int it = 0; it < ITER; ++it) {
            const int t = it * (256 / LP) + tid / LP;
            const T* xp = qkv + (size_t)(t < ntok ? tok0 + t : a.T - 1) * a.qkv_stride + slot * D;
            load8<T>(xp + c0 * 8, x[it][0]); load8<T>(xp + c1 * 8, x[it][1]);
        }
        if (nw) { load8<T>(nw + c0 * 8, g0); load8<T>(nw + c1 * 8, g1); }
#pragma unroll
        for (int it = 0; it < ITER; ++it) {
            const int t = it * (256 / LP) + tid / LP;
            const bool live = t < ntok;
            float (&u)[8] = x[it][0];
            float (&v)[8] = x[it][1];
            if (nw) {
                float ss = 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) ss += u[e] * u[e] + v[e] * v[e];
#pragma unroll
                for (int o = LP / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
                const float inv = 1.f / sqrtf(ss / (float)a.qk_dim + a.eps);
#pragma unroll
                for (int e = 0; e < 8; ++e) { u[e] *= inv * g0[e]; v[e] *= inv * g1[e]; }
            }
            const int pos = a.pos0 + tok0 + t;
            if (!live && is_k && t < nzero) {
#pragma unroll
                for (int e = 0; e < 8; ++e) { u[e] = 0.f; v[e] = 0.f; }
                store8<T>(kc + (size_t)pos * D + c0 * 8, u); store8<T>(kc + (size_t)pos * D + c1 * 8, v);
            }
            if (!live) continue;
            if (rot) {
                const float* cs = a.cos_sin + (size_t)pos * a.rot_dims + k * 8;
                float c[8], s[8];
                load8<float>(cs, c); load8<float>(cs + half8 * 8, s);
#pragma unroll
                for (int e = 0; e < 8; ++e) { const float p = u[e], q = v[e]; u[e] = p * c[e] - q * s[e]; v[e] = q * c[e] + p * s[e]; }
            }
            T* o = is_k ? kc + (size_t)pos * D : qkv + (size_t)(tok0 + t) * a.qkv_stride + slot * D;
            store8<T>(o + c0 * 8, u); store8<T>(o + c1 * 8, v);
        }
        return;
    }
    if (slot < a.n_heads + a.n_kv_heads) {
        float* vec = reinterpret_cast<float*>(smem);     // [VPP][D] normalised vectors of this pass
        const bool is_k = slot >= a.n_heads;
        const int sub = tid % LPV, v = tid / LPV, i0 = sub * 8;
        const T* nw = reinterpret_cast<const T*>(is_k ? a.k_norm : a.q_norm);
        T* kc = reinterpret_cast<T*>(a.K) + (size_t)(is_k ? slot - a.n_heads : 0) * a.s_max * D;
        const int half = a.rot_dims >> 1;
        for (int t0 = 0; t0 < 64; t0 += VPP) {
            const int t = t0 + v;
            const bool live = t < ntok;
            T* xp = qkv + (size_t)(tok0 + (live ? t : 0)) * a.qkv_stride + slot * D + i0;
            float x[8]; load8<T>(xp, x);
            if (nw) {
                float ss = 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
#pragma unroll
                for (int o = LPV / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
                const float inv = 1.f / sqrtf(ss / (float)a.qk_dim + a.eps);
                float g[8]; load8<T>(nw + i0, g);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = x[e] * inv * g[e];
            }
            __syncthreads();                             // the previous pass has been read
            store8<float>(vec + v * D + i0, x);
            __syncthreads();
            const int pos = a.pos0 + tok0 + (live ? t : 0);
            const float* cs = a.cos_sin + (size_t)pos * a.rot_dims;
            if (i0 < a.rot_dims) {
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const int i = i0 + e;
                    if (i >= a.rot_dims) continue;
                    const bool lo = i < half;
                    const int j = lo ? i : i - half;
                    const float p = vec[v * D + (lo ? i + half : i - half)];
                    x[e] = x[e] * cs[j] + (lo ? -p : p) * cs[half + j];
                }
            }
            if (!live) continue;
            store8<T>(is_k ? kc + (size_t)pos * D + i0 : xp, x);
        }
        return;
    }
    // ---- v: [tok][D] -> V^T[d][pos] through LDS (64-key runs) ----
    const int kvh = slot - a.n_heads - a.n_kv_heads;
    constexpr int PITCH = D + 2;
    T* tile = reinterpret_cast<T*>(smem);
    for (int g = tid; g < 64 * (D / 8); g += 256) {
        const int t = g / (D / 8), c = (g % (D / 8)) * 8;
        if (t >= ntok) continue;
        float v[8]; load8<T>(qkv + (size_t)(tok0 + t) * a.qkv_stride + slot * D + c, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) tile[t * PITCH + c + e] = from_f32<T>(v[e]);
    }
    __syncthreads();
    T* vt = reinterpret_cast<T*>(a.VT) + (size_t)kvh * D * a.s_max;
    const int t = tid & 63;
    if (t < ntok || t < nzero) {
        const int pos = a.pos0 + tok0 + t;
        for (int d = tid >> 6; d < D; d += 4) vt[(size_t)d * a.s_max + pos] = t < ntok ? tile[t * PITCH + d] : from_f32<T>(0.f);
    }
}

void launch_qkv_norm_rope_kv(int dtype, int D, const QkvNormRopeArgs& a, hipStream_t st) {
    LMX_REQUIRE(D == 64 || D == 128 || D == 256, "qkv_norm_rope_kv: padded head width must be 64, 128 or 256");
    LMX_REQUIRE(a.qkv_stride % 8 == 0 && a.qkv_stride >= (a.n_heads + 2 * a.n_kv_heads) * D, "qkv_norm_rope_kv: bad row pitch");
    LMX_REQUIRE(a.rot_dims % 2 == 0 && a.rot_dims <= a.qk_dim && a.qk_dim <= D && (a.rot_dims == 0 || a.cos_sin), "qkv_norm_rope_kv: bad rotation");
    LMX_REQUIRE(a.pos0 >= 0 && a.pos0 + a.T <= a.s_max && a.pos0 + a.zero_to <= a.s_max, "qkv_norm_rope_kv: rows past the cache");
    if (a.T <= 0) return;
    const dim3 grid(cdiv(a.zero_to > a.T ? a.zero_to : a.T, 64), a.n_heads + 2 * a.n_kv_heads);
    const bool paired = a.rot_dims % 16 == 0;
    LMX_REQUIRE(a.zero_to == 0 || (paired && a.n_heads == 0), "qkv_norm_rope_kv: clearing is for key / value rows of whole rotation groups");
    size_t smem = (size_t)64 * (D + 2) * dtype_size(dtype);
    if (!paired && smem < 256 * 8 * sizeof(float)) smem = 256 * 8 * sizeof(float);
#define L(TT, DD) do {                                                                                                                   \
        auto kern = paired ? qkv_norm_rope_kv_kernel<TT, DD, true> : qkv_norm_rope_kv_kernel<TT, DD, false>;                                                                                     \
        static bool attr_set[2] = {false, false};                                                                                        \
        if (!attr_set[paired]) { LMX_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, 80 * 1024)); attr_set[paired] = true; } \
        hipLaunchKernelGGL(kern, grid, dim3(256), smem, st, a);                                                                          \
    } while (0)
#define LD(TT) do { if (D == 256) L(TT, 256); else if (D == 128) L(TT, 128); else L(TT, 64); } while (0)
    if (dtype == kBF16) LD(bf16_t); else if (dtype == kF16) LD(f16_t); else LD(float);
#undef LD
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

// softmax end of one (row, head): unnormalised o, sum l and log2-domain maximum M -> output value.  A sink is one more key of score 0 without a value.
__device__ __forceinline__ float softmax_scale(float l, float M, bool sink) {
    if (!sink) return l > 0.f ? 1.f / l : 0.f;
    const float m2 = fmaxf(M, 0.f), f = __builtin_amdgcn_exp2f(M - m2);
    return f / (l * f + __builtin_amdgcn_exp2f(-m2));
}
__device__ __forceinline__ float sigmoid_f32(float g) { return 1.f / (1.f + __expf(-g)); }

// ---------------------------------------------------------------------------------------------------------------
// attention of prompt rows on the vector ALUs: grid (n_heads, rows).  Scores of the row's visible keys wait in LDS.
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int D>
__global__ __launch_bounds__(256) void rows_attn_kernel(FlashArgs a) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float* p_lds = reinterpret_cast<float*>(smem) + 8;       // probabilities of keys [k0, kv_len), k0 = first visible key rounded down to 64
    float* red = reinterpret_cast<float*>(smem);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int head = blockIdx.x, row = blockIdx.y;
    const int kvh = head / (a.n_heads / a.n_kv_heads);
    const int pos = a.q_pos0 + row;
    const int lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
    const int k0 = lo & ~63, nk = ((pos + 1 - k0) + 63) & ~63;
    const T* Q = reinterpret_cast<const T*>(a.Q) + (size_t)row * a.q_stride + head * D;
    const T* Kc = reinterpret_cast<const T*>(a.K) + (size_t)kvh * a.s_max * D;
    const T* Vt = reinterpret_cast<const T*>(a.VT) + (size_t)kvh * D * a.s_max;
    constexpr int LPK = D / 8, KPW = 64 / LPK;
    const float scl = a.scale * 1.4426950408889634f;
    {
        const int sub = lane % LPK, kslot = lane / LPK;
        float qv[8]; load8<T>(Q + sub * 8, qv);
        for (int b = wave * KPW; b < nk; b += 4 * KPW) {
            const int key = k0 + b + kslot;
            float kv[8]; load8<T>(Kc + (size_t)(key <= pos ? key : pos) * D + sub * 8, kv);
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) s = fmaf(qv[e], kv[e], s);
#pragma unroll
            for (int o = LPK / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
            if (sub == 0) p_lds[b + kslot] = key >= lo && key <= pos ? s * scl : -INFINITY;
        }
    }
    __syncthreads();
    float mx = -INFINITY;
    for (int k = tid; k < nk; k += 256) mx = fmaxf(mx, p_lds[k]);
    mx = block_max<4>(mx, red);
    float sum = 0.f;
    for (int k = tid; k < nk; k += 256) { const float e = __builtin_amdgcn_exp2f(p_lds[k] - mx); p_lds[k] = e; sum += e; }
    sum = block_sum<4>(sum, red);
    __syncthreads();
    float out = softmax_scale(sum, mx, a.sink != 0);
    if (a.gate) out *= sigmoid_f32(to_f32(reinterpret_cast<const T*>(a.gate)[(size_t)row * a.q_stride + head]));
    T* O = reinterpret_cast<T*>(a.O) + (size_t)row * a.o_stride + head * D;
    const int sub = tid & 7, drow = tid >> 3;
#pragma unroll
    for (int db = 0; db < D / 32; ++db) {
        const int d = db * 32 + drow;
        float acc = 0.f;
        for (int b = 0; b < nk; b += 64) {
            float vv[8]; load8<T>(Vt + (size_t)d * a.s_max + k0 + b + sub * 8, vv);
            float pv[8]; load8<float>(p_lds + b + sub * 8, pv);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc = fmaf(pv[e], pv[e] != 0.f ? vv[e] : 0.f, acc);
        }
        acc += __shfl_xor(acc, 1, 64); acc += __shfl_xor(acc, 2, 64); acc += __shfl_xor(acc, 4, 64);
        if (sub == 0) O[d] = from_f32<T>(acc * out);
    }
}

void launch_rows_attn(int dtype, int D, const FlashArgs& a, hipStream_t st) {
    LMX_REQUIRE(D == 64 || D == 128 || D == 256, "rows_attn: padded head width must be 64, 128 or 256");
    LMX_REQUIRE(a.s_max % 64 == 0 && a.q_len > 0 && a.q_pos0 >= 0 && a.q_pos0 + a.q_len <= a.s_max, "rows_attn: bad lengths");
    const int last = a.q_pos0 + a.q_len;
    const int span = a.window > 0 && a.window < last ? a.window : last;
    const size_t smem = ((size_t)span + 136) * sizeof(float);
    LMX_REQUIRE(smem <= 160 * 1024, "rows_attn: score row does not fit LDS");
#define L(TT, DD) do {                                                                                                                   \
        auto kern = rows_attn_kernel<TT, DD>;                                                                                            \
        static bool attr_set = false;                                                                                                    \
        if (!attr_set) { LMX_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024)); attr_set = true; } \
        hipLaunchKernelGGL(kern, dim3(a.n_heads, a.q_len), dim3(256), smem, st, a);                                                      \
    } while (0)
#define LD(TT) do { if (D == 256) L(TT, 256); else if (D == 128) L(TT, 128); else L(TT, 64); } while (0)
    if (dtype == kBF16) LD(bf16_t); else if (dtype == kF16) LD(f16_t); else LD(float);
#undef LD
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// one new token per sequence.  grid (n_heads, n_split, sequences), 256 threads.  Split s of n_split walks the 128-key chunks c0 + s, c0 + s + n_split, ... of the
// window [pos - window + 1, pos] with an online softmax; every K / V^T load of a chunk is requested before anything waits, the first chunk's ahead of the query's own
// norm and rotation.  The workgroup that walks the chunk of position `pos` takes the new key from the qkv row (and, for the first query head of a kv group, appends
// it); it is never read back from the cache inside the launch.  Splits are merged by the last workgroup of a head to arrive (write-through partials, one ticket).
// ---------------------------------------------------------------------------------------------------------------
template <typename T> struct Chunk8;
template <> struct Chunk8<bf16_t> {
    uint4 r;
    __device__ __forceinline__ void load(const bf16_t* p) { r = *reinterpret_cast<const uint4*>(p); }
    __device__ __forceinline__ void get(float (&v)[8]) const {
        v[0] = unpack_lo<bf16_t>(r.x); v[1] = unpack_hi<bf16_t>(r.x); v[2] = unpack_lo<bf16_t>(r.y); v[3] = unpack_hi<bf16_t>(r.y);
        v[4] = unpack_lo<bf16_t>(r.z); v[5] = unpack_hi<bf16_t>(r.z); v[6] = unpack_lo<bf16_t>(r.w); v[7] = unpack_hi<bf16_t>(r.w);
    }
};
template <> struct Chunk8<f16_t> {
    uint4 r;
    __device__ __forceinline__ void load(const f16_t* p) { r = *reinterpret_cast<const uint4*>(p); }
    __device__ __forceinline__ void get(float (&v)[8]) const {
        v[0] = unpack_lo<f16_t>(r.x); v[1] = unpack_hi<f16_t>(r.x); v[2] = unpack_lo<f16_t>(r.y); v[3] = unpack_hi<f16_t>(r.y);
        v[4] = unpack_lo<f16_t>(r.z); v[5] = unpack_hi<f16_t>(r.z); v[6] = unpack_lo<f16_t>(r.w); v[7] = unpack_hi<f16_t>(r.w);
    }
};
template <> struct Chunk8<float> {
    float r[8];
    __device__ __forceinline__ void load(const float* p) { load8<float>(p, r); }
    __device__ __forceinline__ void get(float (&v)[8]) const {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = r[e];
    }
};

// one head vector by one wave: norm over the true width, rotation, into out[D] (fp32 LDS); tmp[D] is scratch of this wave
template <typename T, int D>
__device__ __forceinline__ void norm_rope_vec(const T* __restrict__ x, const T* __restrict__ nw, float eps, int qk_dim, const float* __restrict__ cs, int rot_dims,
                                              float* tmp, float* out, int lane) {
    constexpr int E = D / 64;
    float v[E];
#pragma unroll
    for (int j = 0; j < E; ++j) v[j] = to_f32(x[lane + 64 * j]);
    if (nw) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < E; ++j) ss += v[j] * v[j];
        const float inv = 1.f / sqrtf(wave_sum(ss) / (float)qk_dim + eps);
#pragma unroll
        for (int j = 0; j < E; ++j) v[j] = v[j] * inv * to_f32(nw[lane + 64 * j]);
    }
#pragma unroll
    for (int j = 0; j < E; ++j) tmp[lane + 64 * j] = v[j];
    __builtin_amdgcn_wave_barrier();
    const int half = rot_dims >> 1;
#pragma unroll
    for (int j = 0; j < E; ++j) {
        const int i = lane + 64 * j;
        if (i < rot_dims) {
            const bool lo = i < half;
            const int k = lo ? i : i - half;
            const float p = tmp[lo ? i + half : i - half];
            v[j] = v[j] * cs[k] + (lo ? -p : p) * cs[half + k];
        }
        // the same rounding as the prompt's rows: q enters the scores and k the cache in the model dtype
        out[i] = round_to<T>(v[j]);
    }
}

template <typename T, int D>
__global__ __launch_bounds__(256) void decode_win_kernel(WinDecodeArgs a) {
    __shared__ __attribute__((aligned(16))) float sc[DF_CHUNK];
    __shared__ __attribute__((aligned(16))) float qs[D], ks[D];
    __shared__ float tmp[2][D];
    __shared__ float red[8];
    __shared__ float mg_m[DF_MAX_SPLIT], mg_w[DF_MAX_SPLIT];
    __shared__ float mg_o[256];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int head = blockIdx.x, split = blockIdx.y, z = blockIdx.z;
    const DecodeFusedSeq e = a.tab ? a.tab[z] : a.one;
    int pos = a.pos >= 0 ? a.pos : *e.pos_ptr;
    pos = pos < a.s_max ? pos : a.s_max - 1;               // the host keeps len + steps <= s_max; never index past the cache whatever the device word holds
    const int group = a.n_heads / a.n_kv_heads, kvh = head / group;
    const int lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
    const int c0 = lo / DF_CHUNK, c1 = pos / DF_CHUNK;
    const T* row = reinterpret_cast<const T*>(a.qkv) + (size_t)z * a.qkv_stride;
    T* Kc = reinterpret_cast<T*>(e.K) + (size_t)kvh * a.s_max * D;
    T* Vt = reinterpret_cast<T*>(e.VT) + (size_t)kvh * D * a.s_max;
    const T* vnew = row + (a.n_heads + a.n_kv_heads + kvh) * D;
    const float* cs = a.cos_sin + (size_t)pos * a.rot_dims;
    const bool owner = (c1 - c0) % a.n_split == split;      // this workgroup walks the new key's chunk
    constexpr int WS = D + 4;
    float* ws = e.ws + ((size_t)head * a.n_split + split) * WS;

    constexpr int LPK = D / 8, KPW = 64 / LPK, KU = DF_CHUNK / (4 * KPW), DB = D / 32;
    const float scl = a.scale * 1.4426950408889634f;
    const int sub = lane % LPK, kslot = lane / LPK;
    const int s8 = tid & 7, drow = tid >> 3;
    Chunk8<T> kr[KU], vr[2][DB];
    auto load_chunk = [&](int c) {
#pragma unroll
        for (int u = 0; u < KU; ++u) {
            int key = c * DF_CHUNK + (u * 4 + wave) * KPW + kslot;
            key = key < pos ? key : (pos > 0 ? pos - 1 : 0);             // rows past the cached keys re-read the last one; their scores are dropped
            kr[u].load(Kc + (size_t)key * D + sub * 8);
        }
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
            for (int db = 0; db < DB; ++db) vr[kb][db].load(Vt + (size_t)(db * 32 + drow) * a.s_max + c * DF_CHUNK + kb * 64 + s8 * 8);
    };
    if (c0 + split <= c1) load_chunk(c0 + split);
    if (wave == 0) norm_rope_vec<T, D>(row + head * D, reinterpret_cast<const T*>(a.q_norm), a.eps, a.qk_dim, cs, a.rot_dims, tmp[0], qs, lane);
    else if (wave == 1 && owner) norm_rope_vec<T, D>(row + (a.n_heads + kvh) * D, reinterpret_cast<const T*>(a.k_norm), a.eps, a.qk_dim, cs, a.rot_dims, tmp[1], ks, lane);
    __syncthreads();
    if (owner && wave == 0) {
        float s = 0.f;
#pragma unroll
        for (int j = 0; j < D / 64; ++j) s = fmaf(qs[lane + 64 * j], ks[lane + 64 * j], s);
        s = wave_sum(s);
        if (lane == 0) red[6] = s * scl;
    }
    __syncthreads();
    if (owner && head % group == 0) {
        for (int d = tid; d < D; d += 256) {
            Kc[(size_t)pos * D + d] = from_f32<T>(ks[d]);
            Vt[(size_t)d * a.s_max + pos] = vnew[d];
        }
    }
    float qv[8]; load8<float>(qs + sub * 8, qv);
    float m = -INFINITY, l = 0.f, acc[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db) acc[db] = 0.f;
    for (int c = c0 + split; c <= c1; c += a.n_split) {
        const int kb0 = c * DF_CHUNK;
#pragma unroll
        for (int u = 0; u < KU; ++u) {
            const int kl = (u * 4 + wave) * KPW + kslot, key = kb0 + kl;
            float kv[8]; kr[u].get(kv);
            float s = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) s = fmaf(qv[i], kv[i], s);
#pragma unroll
            for (int o = LPK / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
            if (sub == 0) sc[kl] = key == pos ? red[6] : (key >= lo && key < pos ? s * scl : -INFINITY);
        }
        __syncthreads();
        const float s = tid < DF_CHUNK ? sc[tid] : -INFINITY;
        const float m_new = fmaxf(m, block_max<4>(s, red));              // finite: a walked chunk holds at least one visible key
        const float alpha = __builtin_amdgcn_exp2f(m - m_new);           // first chunk: exp2(-inf) = 0 on zero accumulators
        const float ex = __builtin_amdgcn_exp2f(s - m_new);
        l = l * alpha + block_sum<4>(ex, red);
        m = m_new;
        float p_new = 0.f;
        if (c == c1) {                                                   // the newest key's value comes from the row, not from the cache
            if (tid == pos - kb0) red[7] = ex;
            if (tid < DF_CHUNK) sc[tid] = tid == pos - kb0 ? 0.f : ex;
        } else if (tid < DF_CHUNK) sc[tid] = ex;
        __syncthreads();
        if (c == c1) p_new = red[7];
#pragma unroll
        for (int db = 0; db < DB; ++db) acc[db] *= alpha;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            float p[8]; load8<float>(sc + kb * 64 + s8 * 8, p);
#pragma unroll
            for (int db = 0; db < DB; ++db) {
                float v[8]; vr[kb][db].get(v);
#pragma unroll
                for (int i = 0; i < 8; ++i) acc[db] = fmaf(p[i], p[i] != 0.f ? v[i] : 0.f, acc[db]);      // columns outside the window or past the cache never enter, whatever they hold
            }
        }
        if (c == c1 && s8 == 0) {
#pragma unroll
            for (int db = 0; db < DB; ++db) acc[db] = fmaf(p_new, to_f32(vnew[db * 32 + drow]), acc[db]);
        }
        if (c + a.n_split <= c1) load_chunk(c + a.n_split);
        __syncthreads();                                                 // sc is rewritten by the next chunk
    }
    float gate = 1.f;
    if (a.gate_off >= 0) gate = sigmoid_f32(to_f32(row[a.gate_off + head]));
    T* out = reinterpret_cast<T*>(a.out) + (size_t)z * a.out_stride + head * D;
    const float fin = a.n_split == 1 ? softmax_scale(l, m, a.sink != 0) * gate : 0.f;
#pragma unroll
    for (int db = 0; db < DB; ++db) {
        float t = acc[db];
        t += __shfl_xor(t, 1, 64); t += __shfl_xor(t, 2, 64); t += __shfl_xor(t, 4, 64);
        if (s8 == 0) {
            const int d = db * 32 + drow;
            if (a.n_split == 1) out[d] = from_f32<T>(t * fin);
            else __hip_atomic_store(ws + d, t, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        }
    }
    if (a.n_split == 1) return;
    if (tid == 0) {
        __hip_atomic_store(ws + D, m, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __hip_atomic_store(ws + D + 1, l, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    // ---- merge by the last workgroup to arrive for this head (decode_fused_body's protocol: write-through payload, every wave drains, one relaxed ticket) ----
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (tid == 0) red[5] = __hip_atomic_fetch_add(e.counters + head, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == a.n_split - 1 ? 1.f : 0.f;
    __syncthreads();
    if (red[5] == 0.f) return;
    const float* wsh = e.ws + (size_t)head * a.n_split * WS;
    if (tid < a.n_split) {
        mg_m[tid] = __hip_atomic_load(wsh + tid * WS + D, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        mg_w[tid] = __hip_atomic_load(wsh + tid * WS + D + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    constexpr int NG = 256 / D, SPG = DF_MAX_SPLIT / NG;
    const int g = tid / D, d = tid % D;
    float ov[SPG];
#pragma unroll
    for (int i = 0; i < SPG; ++i) {
        const int sp = g + i * NG;
        ov[i] = sp < a.n_split ? __hip_atomic_load(wsh + sp * WS + d, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) : 0.f;
    }
    __syncthreads();
    float M = -INFINITY, lt = 0.f, o = 0.f;
    for (int sp = 0; sp < a.n_split; ++sp) M = fmaxf(M, mg_m[sp]);
    for (int sp = 0; sp < a.n_split; ++sp) lt += __builtin_amdgcn_exp2f(mg_m[sp] - M) * mg_w[sp];          // a split without a chunk left (-inf, 0): weight 0
#pragma unroll
    for (int i = 0; i < SPG; ++i) {
        const int sp = g + i * NG;
        if (sp < a.n_split) o += __builtin_amdgcn_exp2f(mg_m[sp] - M) * ov[i];
    }
    mg_o[tid] = o;
    __syncthreads();
    if (g == 0) {
#pragma unroll
        for (int i = 1; i < NG; ++i) o += mg_o[i * D + d];
        out[d] = from_f32<T>(o * softmax_scale(lt, M, a.sink != 0) * gate);
    }
    if (tid == 0) __hip_atomic_store(e.counters + head, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);    // re-arm for the next launch
}

void launch_decode_win(int dtype, int D, const WinDecodeArgs& a, hipStream_t st) {
    LMX_REQUIRE(D == 64 || D == 128 || D == 256, "decode_win: padded head width must be 64, 128 or 256");
    LMX_REQUIRE(a.s_max % DF_CHUNK == 0 && a.n_split >= 1 && a.n_split <= DF_MAX_SPLIT && a.n_seq >= 1, "decode_win: cache in whole 128-key chunks, 1..32 splits");
    LMX_REQUIRE(a.n_heads >= 1 && a.n_kv_heads >= 1 && a.n_heads % a.n_kv_heads == 0 && a.qkv && a.out, "decode_win: bad arguments");
    LMX_REQUIRE(a.rot_dims % 2 == 0 && a.rot_dims <= a.qk_dim && a.qk_dim <= D && (a.rot_dims == 0 || a.cos_sin), "decode_win: bad rotation");
    LMX_REQUIRE(a.tab || (a.n_seq == 1 && a.one.K && a.one.VT && a.one.ws && a.one.counters && (a.pos >= 0 || a.one.pos_ptr)), "decode_win: bad sequence");
    const dim3 grid(a.n_heads, a.n_split, a.n_seq);
#define L(TT, DD) LMX_LAUNCH((decode_win_kernel<TT, DD>), grid, dim3(256), 0, st, a)
#define LD(TT) do { if (D == 256) L(TT, 256); else if (D == 128) L(TT, 128); else L(TT, 64); } while (0)
    if (dtype == kBF16) LD(bf16_t); else if (dtype == kF16) LD(f16_t); else LD(float);
#undef LD
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

}  // namespace lmx
