// Latent attention (kernels.h: LatentNormArgs, LatentDecodeArgs): a token's keys and values of all heads are linear in one normalised row of R values, the only thing
// the cache holds, [s_max][R].
//
//   latent_norm_kernel     rows of a projection: query latent normalised in place, key / value latent normalised into the cache
//   latent_decode_kernel   one new token per sequence with the queries already taken into the latent space (q W_uk): the cache rows serve as keys and as values
// (A prompt expands the latents its rows can see to per-head keys and values and takes the prompt attention kernels.)
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

void launch_latent_decode(int dtype, const LatentDecodeArgs& a, hipStream_t st) {
    LMX_REQUIRE(a.R == 64 || a.R == 128 || a.R == 256 || a.R == 512, "latent_decode: padded latent width must be 64, 128, 256 or 512");
    LMX_REQUIRE(a.H >= 1 && a.n_split >= 1 && a.n_split <= DF_MAX_SPLIT && a.n_seq >= 1 && a.q && a.out && a.s_max >= 1, "latent_decode: bad arguments");
    LMX_REQUIRE(a.tab || (a.n_seq == 1 && a.one.K && a.one.pos_ptr && a.one.ws && a.one.counters), "latent_decode: bad sequence");
    const dim3 grid(a.H, a.n_split, a.n_seq);
#define L(TT, KK) LMX_LAUNCH((latent_decode_kernel<TT, KK>), grid, dim3(256), 0, st, a)
#define LR(TT) do { if (a.R == 64) L(TT, 8); else if (a.R == 128) L(TT, 16); else if (a.R == 256) L(TT, 32); else L(TT, 64); } while (0)
    if (dtype == kBF16) LR(bf16_t); else if (dtype == kF16) LR(f16_t); else LR(float);
#undef LR
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

}  // namespace lmx
