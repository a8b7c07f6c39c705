// Latent attention (kernels.h: LatentNormArgs, LatentDecodeArgs): a token's keys and values of all heads are linear in one normalised row of R values, the only thing
// the cache holds, [s_max][R].
//
//   latent_norm_kernel     rows of a projection: query latent normalised in place, key / value latent normalised into the cache
//   latent_decode_kernel   one new token per sequence with the queries already taken into the latent space (q W_uk): the cache rows serve as keys and as values
//   latent_mfma_kernel     the same for 16-bit latents of 128 values and more: 16 heads share every cached row they read, both products on MFMA tiles;
//                          latent_merge_kernel joins the splits of a context
// (A prompt expands the latents its rows can see to per-head keys and values and takes the prompt attention kernels.)
#include <algorithm>

#include "common.h"
#include "kernels.h"
#include "attention_decode.h"

namespace lmx {

// grid (rows), 256 threads: waves 0, 1 own the query latent, waves 2, 3 the other one
template <typename T>
__global__ __launch_bounds__(256) void latent_norm_kernel(LatentNormArgs a) {
    __shared__ float red[4];
    const int row = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, half = wave >> 1, lt = tid & 127;
    T* src = reinterpret_cast<T*>(a.proj) + (size_t)row * a.ld + (half ? a.Q : 0);
    const T* w = reinterpret_cast<const T*>(half ? a.r_w : a.q_w);
    const int n = half ? a.R : a.Q;
    T* dst = src;
    if (half) {
        int pos = a.tab ? *a.tab[row].pos_ptr : a.pos_ptr ? *a.pos_ptr : a.pos0 + row;
        pos = pos < a.s_max ? pos : a.s_max - 1;
        dst = reinterpret_cast<T*>(a.tab ? a.tab[row].K : a.cache) + (size_t)pos * a.R;
    }
    float ss = 0.f;
    for (int c = lt * 8; c < n; c += 1024) {
        float v[8]; load8<T>(src + c, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf(v[e], v[e], ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[wave] = ss;
    __syncthreads();
    const float inv = 1.f / sqrtf((red[half * 2] + red[half * 2 + 1]) / (float)(half ? a.r_n : a.q_n) + a.eps);
    for (int c = lt * 8; c < n; c += 1024) {
        float v[8], g[8]; load8<T>(src + c, v); load8<T>(w + c, g);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] *= inv * g[e];
        store8<T>(dst + c, v);
    }
}

void launch_latent_norm(int dtype, const LatentNormArgs& a, int rows, hipStream_t st) {
    LMX_REQUIRE(a.Q % 64 == 0 && a.R % 64 == 0 && a.q_n >= 1 && a.q_n <= a.Q && a.r_n >= 1 && a.r_n <= a.R && a.ld % 8 == 0 && a.ld >= a.Q + a.R, "latent_norm: bad widths");
    LMX_REQUIRE(a.proj && a.q_w && a.r_w && (a.tab || (a.cache && (a.pos_ptr ? rows == 1 : a.pos0 >= 0 && a.pos0 + rows <= a.s_max))), "latent_norm: bad cache rows");
    if (rows <= 0) return;
#define L(TT) LMX_LAUNCH(latent_norm_kernel<TT>, dim3(rows), dim3(256), 0, st, a)
    if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// grid (heads, n_split, sequences), 256 threads.  R / 8 lanes own one key at a time: an online softmax per lane group over the keys it meets (the loaded row is key
// and value), merged across the groups and waves of the workgroup and, with splits, by the last workgroup of a head to arrive (decode_win_kernel's protocol).
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int LPK>
__global__ __launch_bounds__(256) void latent_decode_kernel(LatentDecodeArgs a) {
    constexpr int R = LPK * 8, GPW = 64 / LPK, NS = 4 * GPW, U = 4;      // streams of a workgroup, keys of a stream in flight
    __shared__ __attribute__((aligned(16))) float ms[NS], ls[NS];
    __shared__ __attribute__((aligned(16))) float os[NS][R];
    __shared__ float mg_m[DF_MAX_SPLIT], mg_w[DF_MAX_SPLIT];
    __shared__ int last_s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int head = blockIdx.x, split = blockIdx.y, z = blockIdx.z;
    const DecodeFusedSeq e = a.tab ? a.tab[z] : a.one;
    int pos = *e.pos_ptr;
    pos = pos < a.s_max ? pos : a.s_max - 1;
    const int lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
    const T* cache = reinterpret_cast<const T*>(e.K);
    const int sub = lane % LPK, strm = wave * GPW + lane / LPK;
    const size_t row = ((size_t)z * a.H + head) * R;
    float q[8]; load8<T>(reinterpret_cast<const T*>(a.q) + row + sub * 8, q);
    const float scl = a.scale * 1.4426950408889634f;
    float m = -INFINITY, l = 0.f, acc[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i] = 0.f;
    const int step = a.n_split * NS;
    for (int j0 = lo + split * NS + strm; j0 - strm <= pos; j0 += step * U) {          // wave-uniform trip count
        float c[U][8], s[U];
        float mx = m;
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int j = j0 + u * step;
            load8<T>(cache + (size_t)(j <= pos ? j : pos) * R + sub * 8, c[u]);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            float t = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) t = fmaf(q[i], c[u][i], t);
#pragma unroll
            for (int o = LPK / 2; o > 0; o >>= 1) t += __shfl_xor(t, o, 64);
            s[u] = j0 + u * step <= pos ? t * scl : -INFINITY;
            mx = fmaxf(mx, s[u]);
        }
        const float alpha = mx == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m - mx);
        l *= alpha;
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[i] *= alpha;
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const float p = mx == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(s[u] - mx);
            l += p;
#pragma unroll
            for (int i = 0; i < 8; ++i) acc[i] = fmaf(p, c[u][i], acc[i]);
        }
        m = mx;
    }
    if (sub == 0) { ms[strm] = m; ls[strm] = l; }
    store8<float>(&os[strm][sub * 8], acc);
    __syncthreads();
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int i = 0; i < NS; ++i) M = fmaxf(M, ms[i]);
    if (M != -INFINITY) {
#pragma unroll
        for (int i = 0; i < NS; ++i) L += __builtin_amdgcn_exp2f(ms[i] - M) * ls[i];
    }
    T* out = reinterpret_cast<T*>(a.out) + row;
    float* ws = a.n_split > 1 ? e.ws + (size_t)head * a.n_split * (R + 4) : nullptr;
    for (int d = tid; d < R; d += 256) {
        float o = 0.f;
        if (M != -INFINITY) {
#pragma unroll
            for (int i = 0; i < NS; ++i) o = fmaf(__builtin_amdgcn_exp2f(ms[i] - M), os[i][d], o);
        }
        if (a.n_split == 1) out[d] = from_f32<T>(o / L);
        else __hip_atomic_store(ws + split * (R + 4) + d, o, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    if (a.n_split == 1) return;
    if (tid == 0) {
        __hip_atomic_store(ws + split * (R + 4) + R, M, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __hip_atomic_store(ws + split * (R + 4) + R + 1, L, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (tid == 0) last_s = __hip_atomic_fetch_add(e.counters + head, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == a.n_split - 1;
    __syncthreads();
    if (!last_s) return;
    if (tid < a.n_split) {
        mg_m[tid] = __hip_atomic_load(ws + tid * (R + 4) + R, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        mg_w[tid] = __hip_atomic_load(ws + tid * (R + 4) + R + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    __syncthreads();
    M = -INFINITY; L = 0.f;
    for (int i = 0; i < a.n_split; ++i) M = fmaxf(M, mg_m[i]);
    for (int i = 0; i < a.n_split; ++i) L += __builtin_amdgcn_exp2f(mg_m[i] - M) * mg_w[i];      // a split without a key left (-inf, 0): weight 0
    for (int d = tid; d < R; d += 256) {
        float o = 0.f;
        for (int i = 0; i < a.n_split; ++i) o = fmaf(__builtin_amdgcn_exp2f(mg_m[i] - M), __hip_atomic_load(ws + i * (R + 4) + d, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT), o);
        out[d] = from_f32<T>(o / L);
    }
    if (tid == 0) __hip_atomic_store(e.counters + head, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);      // re-arm for the next launch
}

// ---------------------------------------------------------------------------------------------------------------
// grid (n_split, ceil(heads / 16), sequences), 256 threads; tiles of 128 keys, every n_split-th tile a workgroup's.
//   scores   wave w: 32 keys of the tile, 16 heads x 16 keys per product chain over R; they meet in LDS (fp32)
//   softmax  every wave, redundantly: lane l holds head l % 16 and keys 8 (l / 16) .. + 7 of each 32, which is the A operand of the second product
//   output   wave w: column blocks of 128 values w, w + 4, ...  A lane loads 8 cached rows x 8 values and turns them in registers (packed halves of two rows), so its eight
//            B operands are the columns 8 (l % 16) + e of the block
// ---------------------------------------------------------------------------------------------------------------
template <typename T> __device__ __forceinline__ f32x4 mfma16(const uint4& a, const uint4& b, const f32x4& c);
template <> __device__ __forceinline__ f32x4 mfma16<bf16_t>(const uint4& a, const uint4& b, const f32x4& c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_v, a), __builtin_bit_cast(bf16x8_v, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ f32x4 mfma16<f16_t>(const uint4& a, const uint4& b, const f32x4& c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8_v, a), __builtin_bit_cast(f16x8_v, b), c, 0, 0, 0);
}

template <typename T, int R>
__global__ __launch_bounds__(256, 1) void latent_mfma_kernel(LatentDecodeArgs a) {
    static_assert(R <= 512, "one column block per wave");
    constexpr int KT = 128, PITCH = KT + 4, NQ = R / 32;
    __shared__ __attribute__((aligned(16))) float ss[2][16][PITCH];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int split = blockIdx.x, h0 = blockIdx.y * 16, z = blockIdx.z, l16 = lane & 15, g = lane >> 4;
    const int nh = a.H - h0 < 16 ? a.H - h0 : 16;            // heads of this workgroup
    const bool mine = wave * 128 < R;                        // this wave has output columns
    const DecodeFusedSeq e = a.tab ? a.tab[z] : a.one;
    int pos = *e.pos_ptr;
    pos = pos < a.s_max ? pos : a.s_max - 1;
    const int lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
    const T* cache = reinterpret_cast<const T*>(e.K);
    const T* qrow = reinterpret_cast<const T*>(a.q) + ((size_t)z * a.H + h0 + (l16 < nh ? l16 : nh - 1)) * R + g * 8;
    uint4 qf[NQ];
#pragma unroll
    for (int k = 0; k < NQ; ++k) qf[k] = *reinterpret_cast<const uint4*>(qrow + k * 32);
    const float scl = a.scale * 1.4426950408889634f;
    float m = -INFINITY, l = 0.f;
    f32x4 acc[8];
#pragma unroll
    for (int c = 0; c < 8; ++c) acc[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    auto row_at = [&](int j) { return cache + (size_t)(j <= pos ? j : pos) * R; };
    int par = 0;
    for (int base = lo + split * KT; base <= pos; base += a.n_split * KT, par ^= 1) {      // workgroup-uniform
        uint4 kf[2][NQ], r[4][8];
#pragma unroll
        for (int nt = 0; nt < 2; ++nt)
#pragma unroll
            for (int k = 0; k < NQ; ++k) kf[nt][k] = *reinterpret_cast<const uint4*>(row_at(base + wave * 32 + nt * 16 + l16) + g * 8 + k * 32);
        if (mine) {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int i = 0; i < 8; ++i) r[t][i] = *reinterpret_cast<const uint4*>(row_at(base + t * 32 + g * 8 + i) + wave * 128 + l16 * 8);
        }
        f32x4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int k = 0; k < NQ; ++k) { s[0] = mfma16<T>(qf[k], kf[0][k], s[0]); s[1] = mfma16<T>(qf[k], kf[1][k], s[1]); }
#pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
            const int kk = wave * 32 + nt * 16 + l16;
            const bool seen = base + kk <= pos;
#pragma unroll
            for (int i = 0; i < 4; ++i) ss[par][g * 4 + i][kk] = seen ? s[nt][i] * scl : -INFINITY;
        }
        // LDS only: a full barrier would also wait for the rows that are on their way
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        float p[4][8], mx = m;
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            load8<float>(&ss[par][l16][t * 32 + g * 8], p[t]);
#pragma unroll
            for (int i = 0; i < 8; ++i) mx = fmaxf(mx, p[t][i]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64)); mx = fmaxf(mx, __shfl_xor(mx, 32, 64));      // finite: the tile's first key is seen
        const float alpha = __builtin_amdgcn_exp2f(m - mx);
        m = mx; l *= alpha;
        uint4 pf[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) {
#pragma unroll
            for (int i = 0; i < 8; ++i) { p[t][i] = __builtin_amdgcn_exp2f(p[t][i] - mx); l += p[t][i]; }
            pf[t] = uint4{pack2<T>(p[t][0], p[t][1]), pack2<T>(p[t][2], p[t][3]), pack2<T>(p[t][4], p[t][5]), pack2<T>(p[t][6], p[t][7])};
        }
        float al[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) al[i] = __shfl(alpha, g * 4 + i, 64);
        if (!mine) continue;
#pragma unroll
        for (int c = 0; c < 8; ++c) {
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[c][i] *= al[i];
            const unsigned sel = c & 1 ? 0x07060302u : 0x05040100u;      // high or low halves of a pair of rows
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                auto word = [&](int i) { const unsigned w[4] = {r[t][i].x, r[t][i].y, r[t][i].z, r[t][i].w}; return w[c >> 1]; };
                const uint4 f = {__builtin_amdgcn_perm(word(1), word(0), sel), __builtin_amdgcn_perm(word(3), word(2), sel),
                                 __builtin_amdgcn_perm(word(5), word(4), sel), __builtin_amdgcn_perm(word(7), word(6), sel)};
                acc[c] = mfma16<T>(pf[t], f, acc[c]);
            }
        }
    }
    l += __shfl_xor(l, 16, 64); l += __shfl_xor(l, 32, 64);
    // one split: the output; several: accumulators [head][split][R + 4] with maximum and sum behind them, for latent_merge_kernel
    T* out = reinterpret_cast<T*>(a.out) + ((size_t)z * a.H + h0) * R;
    float* ws = a.n_split > 1 ? e.ws + ((size_t)h0 * a.n_split + split) * (R + 4) : nullptr;
    const size_t head = (size_t)a.n_split * (R + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int h = g * 4 + i, c0 = wave * 128 + l16 * 8;
        const float inv = a.n_split == 1 ? 1.f / __shfl(l, h, 64) : 1.f;
        if (h >= nh || !mine) continue;
        float v[8];
#pragma unroll
        for (int c = 0; c < 8; ++c) v[c] = acc[c][i] * inv;
        if (a.n_split == 1) store8<T>(out + (size_t)h * R + c0, v); else store8<float>(ws + h * head + c0, v);
    }
    if (a.n_split > 1 && tid < nh) { ws[tid * head + R] = m; ws[tid * head + R + 1] = l; }
}

// grid (heads, sequences), R / 4 threads
template <typename T, int R>
__global__ __launch_bounds__(R / 4) void latent_merge_kernel(LatentDecodeArgs a) {
    const DecodeFusedSeq e = a.tab ? a.tab[blockIdx.y] : a.one;
    const float* ws = e.ws + (size_t)blockIdx.x * a.n_split * (R + 4);
    const int d = threadIdx.x * 4;
    float M = -INFINITY, L = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < a.n_split; ++i) M = fmaxf(M, ws[i * (R + 4) + R]);
#pragma unroll 8
    for (int i = 0; i < a.n_split; ++i) {                    // a split without a key (-inf, 0) has weight 0
        const float4 v = *reinterpret_cast<const float4*>(ws + i * (R + 4) + d);
        const float w = __builtin_amdgcn_exp2f(ws[i * (R + 4) + R] - M);
        L = fmaf(w, ws[i * (R + 4) + R + 1], L);
        o[0] = fmaf(w, v.x, o[0]); o[1] = fmaf(w, v.y, o[1]); o[2] = fmaf(w, v.z, o[2]); o[3] = fmaf(w, v.w, o[3]);
    }
    const float inv = 1.f / L;
    T* out = reinterpret_cast<T*>(a.out) + ((size_t)blockIdx.y * a.H + blockIdx.x) * R + d;
#pragma unroll
    for (int c = 0; c < 4; ++c) out[c] = from_f32<T>(o[c] * inv);
}

// workgroups along a context of `span` keys: enough of them to fill the chip, no more
static bool latent_mfma(int dtype, int R) { return dtype != kF32 && R >= 128; }
int latent_decode_split(int dtype, int R, int H, int n_seq, int span) {
    const bool mf = latent_mfma(dtype, R);
    const int wgs = mf ? cdiv(H, 16) * n_seq : H * n_seq;
    return std::max(1, std::min(std::min(cdiv(span, mf ? 128 : 64), 32), cdiv(mf ? 256 : 1024, wgs)));
}

void launch_latent_decode(int dtype, const LatentDecodeArgs& a, hipStream_t st) {
    LMX_REQUIRE(a.R == 64 || a.R == 128 || a.R == 256 || a.R == 512, "latent_decode: padded latent width must be 64, 128, 256 or 512");
    LMX_REQUIRE(a.H >= 1 && a.n_split >= 1 && a.n_split <= DF_MAX_SPLIT && a.n_seq >= 1 && a.q && a.out && a.s_max >= 1, "latent_decode: bad arguments");
    LMX_REQUIRE(a.tab || (a.n_seq == 1 && a.one.K && a.one.pos_ptr && a.one.ws && a.one.counters), "latent_decode: bad sequence");
    if (latent_mfma(dtype, a.R)) {
        const dim3 grid(a.n_split, cdiv(a.H, 16), a.n_seq);
#define M1(TT, RR) do { LMX_LAUNCH((latent_mfma_kernel<TT, RR>), grid, dim3(256), 0, st, a); if (a.n_split > 1) LMX_LAUNCH((latent_merge_kernel<TT, RR>), dim3(a.H, a.n_seq), dim3(RR / 4), 0, st, a); } while (0)
#define M(TT) do { if (a.R == 128) M1(TT, 128); else if (a.R == 256) M1(TT, 256); else M1(TT, 512); } while (0)
        if (dtype == kBF16) M(bf16_t); else M(f16_t);
#undef M
#undef M1
        LMX_CHECK_HIP(hipGetLastError());
        return;
    }
    const dim3 grid(a.H, a.n_split, a.n_seq);
#define L(TT, KK) LMX_LAUNCH((latent_decode_kernel<TT, KK>), grid, dim3(256), 0, st, a)
#define LR(TT) do { if (a.R == 64) L(TT, 8); else if (a.R == 128) L(TT, 16); else if (a.R == 256) L(TT, 32); else L(TT, 64); } while (0)
    if (dtype == kBF16) LR(bf16_t); else if (dtype == kF16) LR(f16_t); else LR(float);
#undef LR
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

}  // namespace lmx
