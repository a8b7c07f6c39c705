// Grouped linears and mixtures of experts.
//
//   moe_router_kernel    fp32 router logits, the `top` largest and the softmax over them
//   group_gemv_kernel    one row through the weight of its group (an expert, or a head), weights streamed straight into the vector ALUs
#include "common.h"
#include "kernels.h"
#include "gemm_common.h"

namespace lmx {

constexpr int MOE_MAX_E = 256, MOE_MAX_TOP = 32;

// one wave: the `top` largest of z[0, E) (lowest index first among equals) and their softmax
__device__ __forceinline__ void pick_top(const float* z, int E, int top, int lane, int* ids, float* wt) {
    float v[MOE_MAX_E / 64];
#pragma unroll
    for (int i = 0; i < MOE_MAX_E / 64; ++i) v[i] = lane + 64 * i < E ? z[lane + 64 * i] : -INFINITY;
    float mine = 0.f, zmax = 0.f; int my_id = 0;            // lane k keeps pick k
    for (int k = 0; k < top; ++k) {
        float b = -INFINITY; int bi = 0x7fffffff;
#pragma unroll
        for (int i = 0; i < MOE_MAX_E / 64; ++i) if (v[i] > b) { b = v[i]; bi = lane + 64 * i; }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(b, o, 64); const int oi = __shfl_xor(bi, o, 64);
            if (ob > b || (ob == b && oi < bi)) { b = ob; bi = oi; }
        }
        if (bi >= E) bi = 0;                                 // only non-finite logits leave nothing to pick
        if (k == 0) zmax = b;
        if (lane == k) { mine = b; my_id = bi; }
#pragma unroll
        for (int i = 0; i < MOE_MAX_E / 64; ++i) if (lane + 64 * i == bi) v[i] = -INFINITY;
    }
    const float e = lane < top ? expf(mine - zmax) : 0.f;
    const float sum = wave_sum(e);
    if (lane < top) { ids[lane] = my_id; wt[lane] = e / sum; }
}

// grid (rows), 256 threads
template <typename T>
__global__ __launch_bounds__(256) void moe_router_kernel(MoeRouterArgs a) {
    __shared__ float z[MOE_MAX_E];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const T* x = reinterpret_cast<const T*>(a.x) + (size_t)blockIdx.x * a.ldx;
    for (int e = wave; e < a.E; e += 4) {
        const T* w = reinterpret_cast<const T*>(a.w) + (size_t)e * a.K;
        float s = 0.f;
        for (int c = lane * 8; c < a.K; c += 512) {
            float f[8], v[8]; load8<T>(w + c, f); load8<T>(x + c, v);
#pragma unroll
            for (int i = 0; i < 8; ++i) s = fmaf(f[i], v[i], s);
        }
        s = wave_sum(s);
        if (lane == 0) z[e] = s + (a.bias ? to_f32(reinterpret_cast<const T*>(a.bias)[e]) : 0.f);
    }
    __syncthreads();
    if (wave == 0) pick_top(z, a.E, a.top, lane, a.ids + (size_t)blockIdx.x * a.top, a.wt + (size_t)blockIdx.x * a.top);
}

void launch_moe_router(int dtype, const MoeRouterArgs& a, int rows, hipStream_t st) {
    LMX_REQUIRE(a.E >= 1 && a.E <= MOE_MAX_E && a.top >= 1 && a.top <= a.E && a.top <= MOE_MAX_TOP, "moe_router: 1..256 experts, at most 32 of them per row");
    LMX_REQUIRE(a.K % 8 == 0 && a.ldx % 8 == 0 && a.x && a.w && a.ids && a.wt, "moe_router: bad arguments");
    if (rows <= 0) return;
#define L(TT) LMX_LAUNCH(moe_router_kernel<TT>, dim3(rows), dim3(256), 0, st, a)
    if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// grid (slots, ceil(outputs / outputs per workgroup)), 256 threads.  `lpr` lanes own one weight row (a power of two with 8 lpr <= K): short rows leave no lane idle.
// Gated: a lane group takes the gate row and the up row of its output.
// ---------------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void group_gemv_kernel(GroupGemvArgs a, int lpr, int opw) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* xs = reinterpret_cast<T*>(smem);
    const int tid = threadIdx.x, slot = blockIdx.x;
    const int grp = a.ids ? a.ids[slot] : slot % a.groups;
    const size_t xr = a.ids ? slot / a.per_row : slot / a.groups, cr = a.ids ? slot : slot / a.groups;
    const T* x = reinterpret_cast<const T*>(a.X) + xr * a.ldx + (a.ids ? 0 : grp * a.x_group);
    const T* W = reinterpret_cast<const T*>(a.W) + (size_t)grp * a.w_group;
    T* C = reinterpret_cast<T*>(a.C) + cr * a.ldc + (a.ids ? 0 : grp * a.c_group);
    for (int c = tid * 8; c < a.K; c += 2048) { float v[8]; load8<T>(x + c, v); store8<T>(xs + c, v); }
    __syncthreads();
    const bool gated = act_gated(a.act);
    const int outs = gated ? a.N / 2 : a.N, sub = tid % lpr, per = 256 / lpr;
    const int o0 = blockIdx.y * opw, o1 = o0 + opw < outs ? o0 + opw : outs;
    for (int ob = o0; ob < o1; ob += per) {                  // every lane stays: the sums run over whole lane groups
        const int o = ob + tid / lpr, oc = o < o1 ? o : o1 - 1;
        const int r0 = gated ? 64 * (oc >> 5) + (oc & 31) : oc;
        const T* w0 = W + (size_t)r0 * a.ldw;
        const T* w1 = w0 + (size_t)32 * a.ldw;
        float s0 = 0.f, s1 = 0.f;
        for (int c = sub * 8; c < a.K; c += lpr * 8) {
            float v[8], f[8]; load8<T>(xs + c, v); load8<T>(w0 + c, f);
#pragma unroll
            for (int i = 0; i < 8; ++i) s0 = fmaf(f[i], v[i], s0);
            if (gated) {
                load8<T>(w1 + c, f);
#pragma unroll
                for (int i = 0; i < 8; ++i) s1 = fmaf(f[i], v[i], s1);
            }
        }
        for (int d = lpr >> 1; d > 0; d >>= 1) { s0 += __shfl_xor(s0, d, 64); if (gated) s1 += __shfl_xor(s1, d, 64); }
        if (sub == 0 && o < o1) C[o] = from_f32<T>(gated ? gate_mul(a.act, s0, s1) : s0);
    }
}

void launch_group_gemv(int dtype, const GroupGemvArgs& a, int slots, hipStream_t st) {
    LMX_REQUIRE(a.X && a.W && a.C && a.N >= 1 && a.K >= 64 && a.K % 8 == 0 && a.ldx % 8 == 0 && a.ldw % 8 == 0 && a.w_group % 8 == 0 && a.x_group % 8 == 0, "group_gemv: bad arguments");
    LMX_REQUIRE(!act_gated(a.act) || a.N % 64 == 0, "group_gemv: gated rows come in groups of 64");
    LMX_REQUIRE(a.per_row >= 1 && a.groups >= 1 && (size_t)a.K * dtype_size(dtype) <= 64 * 1024, "group_gemv: bad groups");
    if (slots <= 0) return;
    int lpr = 64;
    while (lpr > 1 && lpr * 8 > a.K) lpr >>= 1;
    const int outs = act_gated(a.act) ? a.N / 2 : a.N, per = 256 / lpr;
    int opw = per;                                           // outputs of a workgroup: more of them while the grid stays large enough
    while (opw < 64 && (long)slots * cdiv(outs, opw * 2) >= 1024) opw *= 2;
    const dim3 grid(slots, cdiv(outs, opw));
#define L(TT) LMX_LAUNCH(group_gemv_kernel<TT>, grid, dim3(256), (size_t)a.K * sizeof(TT), st, a, lpr, opw)
    if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

}  // namespace lmx
