// Grouped linears and mixtures of experts.
//
//   moe_router_kernel    fp32 router logits, the `top` largest and the softmax over them
//   group_plan_kernel    rows of every expert side by side, cut into tiles
//   group_gemm_kernel    the rows of a group times its weight on MFMA tiles (16-bit)
//   group_gemv_kernel    one row through the weight of its group (an expert, or a head), weights streamed straight into the vector ALUs
#include <algorithm>

#include "common.h"
#include "kernels.h"
#include "gemm_common.h"

namespace lmx {

constexpr int MOE_MAX_E = 256, MOE_MAX_TOP = 32;

// the `top` largest of z[0, E) (lowest index first among equals) and their softmax, by one wave: an expert's place is the number of experts ahead of it.
// z is padded with -inf to a multiple of 4
__device__ __forceinline__ void pick_top(const float* z, int E, int top, int lane, int* place, int* ids, float* wt) {
    float v[MOE_MAX_E / 64]; int rank[MOE_MAX_E / 64];
    if (lane < top) place[lane] = lane;                      // only non-finite logits leave a place empty
#pragma unroll
    for (int i = 0; i < MOE_MAX_E / 64; ++i) { v[i] = lane + 64 * i < E ? z[lane + 64 * i] : -INFINITY; rank[i] = 0; }
    for (int j = 0; j < E; j += 4) {
        const float4 q = *reinterpret_cast<const float4*>(z + j);
        const float o[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
        for (int n = 0; n < 4; ++n)
#pragma unroll
            for (int i = 0; i < MOE_MAX_E / 64; ++i) rank[i] += o[n] > v[i] || (o[n] == v[i] && j + n < lane + 64 * i);
    }
#pragma unroll
    for (int i = 0; i < MOE_MAX_E / 64; ++i) if (lane + 64 * i < E && rank[i] < top) place[rank[i]] = lane + 64 * i;
    __builtin_amdgcn_wave_barrier();
    const int id = lane < top ? place[lane] : 0;
    const float e = lane < top ? expf(z[id] - z[place[0]]) : 0.f;
    const float sum = wave_sum(e);
    if (lane < top) { ids[lane] = id; wt[lane] = e / sum; }
}

// grid (rows), 64 NW threads: a wave per expert at a time
template <typename T, int NW>
__global__ __launch_bounds__(64 * NW) void moe_router_kernel(MoeRouterArgs a) {
    __shared__ __attribute__((aligned(16))) float z[MOE_MAX_E];
    __shared__ int place[MOE_MAX_TOP];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const T* x = reinterpret_cast<const T*>(a.x) + (size_t)blockIdx.x * a.ldx;
    if (tid < MOE_MAX_E && tid >= a.E) z[tid] = -INFINITY;
    for (int e = wave; e < a.E; e += NW) {
        const T* w = reinterpret_cast<const T*>(a.w) + (size_t)e * a.K;
        float s = 0.f;
#pragma unroll 4
        for (int c = lane * 8; c < a.K; c += 512) {
            float f[8], v[8]; load8<T>(w + c, f); load8<T>(x + c, v);
#pragma unroll
            for (int i = 0; i < 8; ++i) s = fmaf(f[i], v[i], s);
        }
        s = wave_sum(s);
        if (lane == 0) z[e] = s + (a.bias ? to_f32(reinterpret_cast<const T*>(a.bias)[e]) : 0.f);
    }
    __syncthreads();
    if (wave == 0) pick_top(z, a.E, a.top, lane, place, a.ids + (size_t)blockIdx.x * a.top, a.wt + (size_t)blockIdx.x * a.top);
}

void launch_moe_router(int dtype, const MoeRouterArgs& a, int rows, hipStream_t st) {
    LMX_REQUIRE(a.E >= 1 && a.E <= MOE_MAX_E && a.top >= 1 && a.top <= a.E && a.top <= MOE_MAX_TOP, "moe_router: 1..256 experts, at most 32 of them per row");
    LMX_REQUIRE(a.K % 8 == 0 && a.ldx % 8 == 0 && a.x && a.w && a.ids && a.wt, "moe_router: bad arguments");
    if (rows <= 0) return;
#define L(TT) do { if (rows <= 64) LMX_LAUNCH((moe_router_kernel<TT, 16>), dim3(rows), dim3(1024), 0, st, a); else LMX_LAUNCH((moe_router_kernel<TT, 4>), dim3(rows), dim3(256), 0, st, a); } while (0)
    if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// plan of a grouped product: slots sorted by expert (order) and the tiles of `bm` rows they make.  One workgroup
// ---------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(1024) void group_plan_kernel(const int* ids, int slots, int E, int bm, GroupPlan p) {
    __shared__ int cnt[MOE_MAX_E], pos[MOE_MAX_E], scan[2][MOE_MAX_E], tsum[2][MOE_MAX_E];
    const int tid = threadIdx.x;
    if (tid < MOE_MAX_E) cnt[tid] = 0;
    __syncthreads();
    for (int i = tid; i < slots; i += 1024) atomicAdd(&cnt[ids[i]], 1);
    __syncthreads();
    if (tid < MOE_MAX_E) { scan[0][tid] = cnt[tid]; tsum[0][tid] = (cnt[tid] + bm - 1) / bm; }
    __syncthreads();
    int b = 0;
    for (int o = 1; o < MOE_MAX_E; o <<= 1, b ^= 1) {
        if (tid < MOE_MAX_E) {
            scan[b ^ 1][tid] = scan[b][tid] + (tid >= o ? scan[b][tid - o] : 0);
            tsum[b ^ 1][tid] = tsum[b][tid] + (tid >= o ? tsum[b][tid - o] : 0);
        }
        __syncthreads();
    }
    if (tid < E) {
        const int n = cnt[tid], nt = (n + bm - 1) / bm, r0 = scan[b][tid] - n, t0 = tsum[b][tid] - nt;
        pos[tid] = r0;
        for (int t = 0; t < nt; ++t) p.tiles[t0 + t] = GroupTile{tid, r0 + t * bm, n - t * bm < bm ? n - t * bm : bm, t0, nt, {0, 0, 0}};
    }
    if (tid == MOE_MAX_E - 1) *p.n_tiles = tsum[b][tid];
    __syncthreads();
    for (int i = tid; i < slots; i += 1024) p.order[atomicAdd(&pos[ids[i]], 1)] = i;
}

size_t group_plan_bytes(int slots) { return 256 + ((size_t)slots * 4 + 255) / 256 * 256 + ((size_t)slots / GROUP_MIN_BM + MOE_MAX_E + 1) * sizeof(GroupTile); }
GroupPlan group_plan_at(void* base, int slots) {
    char* p = static_cast<char*>(base);
    return GroupPlan{reinterpret_cast<int*>(p + 256), reinterpret_cast<GroupTile*>(p + 256 + ((size_t)slots * 4 + 255) / 256 * 256), reinterpret_cast<int*>(p)};
}
// rows of a tile: what an average group fills
int group_gemm_bm(int slots, int groups) {
    const int avg = slots / groups;
    return avg <= 24 ? 32 : avg <= 96 ? 64 : avg <= 160 ? 128 : 256;
}
bool group_gemm_applies(int dtype, int slots, int groups) { return dtype != kF32 && slots >= 16 && slots >= groups; }
void launch_group_plan(const int* ids, int slots, int E, int bm, const GroupPlan& p, hipStream_t st) {
    LMX_REQUIRE(ids && slots >= 1 && E >= 1 && E <= MOE_MAX_E && bm >= GROUP_MIN_BM && p.order && p.tiles && p.n_tiles, "group_plan: bad arguments");
    LMX_LAUNCH(group_plan_kernel, dim3(1), dim3(1024), 0, st, ids, slots, E, bm, p);
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// MFMA tiles of a grouped product: the LDS ring of gemm_pipe_kernel (gemm.hip) with a row list.  Logical tiles run group by group, a group's row tiles next to each
// other for one panel of its weight.  The grid is an upper bound: workgroups past the plan's tile count leave at once.
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int BM, int BN, int WM, int WN, int NSTAGE>
__global__ __launch_bounds__(WM * WN * 64) void group_gemm_kernel(GroupGemmArgs a) {
    constexpr int NW = WM * WN, TM = BM / WM, TN = BN / WN, MT = TM / 32, NTL = TN / 32, PIECES = (BM + BN) / 8, PPW = PIECES / NW;
    constexpr int BUF_BYTES = (BM + BN) * GEMM_ROWB;
    static_assert(PIECES % NW == 0 && NTL % 2 == 0 && NSTAGE >= 2 && NSTAGE <= 4 && (NSTAGE - 2) * PPW <= 63, "tile");
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = wave / WN, wn = wave % WN, hi = lane >> 5, l31 = lane & 31;
    const int nt = (a.N + BN - 1) / BN;
    int grp, row0, rows, tile_n;
    if (a.plan.n_tiles) {
        const int total = *a.plan.n_tiles * nt;
        if ((int)blockIdx.x >= total) return;
        const int lid = xcd_remap(blockIdx.x, total);
        const GroupTile t = a.plan.tiles[lid / nt];
        const int rel = lid - t.first * nt;
        const GroupTile u = a.plan.tiles[t.first + rel % t.n_tiles];
        grp = u.group; row0 = u.row0; rows = u.rows; tile_n = rel / t.n_tiles;
    } else {
        const int mt = (a.rows + BM - 1) / BM, lid = xcd_remap(blockIdx.x, a.groups * mt * nt), rel = lid % (mt * nt);
        grp = lid / (mt * nt); tile_n = rel / mt; row0 = rel % mt * BM;
        rows = a.rows - row0 < BM ? a.rows - row0 : BM;
    }
    grp = __builtin_amdgcn_readfirstlane(grp); row0 = __builtin_amdgcn_readfirstlane(row0); rows = __builtin_amdgcn_readfirstlane(rows); tile_n = __builtin_amdgcn_readfirstlane(tile_n);
    const int n0 = tile_n * BN;
    const T* X = reinterpret_cast<const T*>(a.X) + (size_t)grp * a.x_group;
    const T* W = reinterpret_cast<const T*>(a.W) + (size_t)grp * a.w_group;
    const T* gsrc[PPW];
#pragma unroll
    for (int i = 0; i < PPW; ++i) {
        const int row = (wave + NW * i) * 8 + (lane >> 3), chunk = ((lane & 7) ^ (row >> 1)) & 7;
        if (row < BM) {
            int m = row0 + (row < rows ? row : rows - 1);
            if (a.plan.order) m = a.plan.order[m] / a.per_row;
            gsrc[i] = X + (size_t)m * a.ldx + chunk * 8;
        } else {
            int n = n0 + row - BM; n = n < a.N ? n : a.N - 1;
            gsrc[i] = W + (size_t)n * a.ldw + chunk * 8;
        }
    }
    f32x16 acc[NTL][MT];
#pragma unroll
    for (int i = 0; i < NTL; ++i)
#pragma unroll
        for (int j = 0; j < MT; ++j)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;
    const int nk = a.K / GEMM_BK;
    const unsigned lds_base = (unsigned)(uintptr_t)(__attribute__((address_space(3))) char*)smem;
    auto stage = [&](int kt, unsigned buf_off) {             // (inline asm for the reason given in gemm_pipe_kernel: ordering is the counted vmcnt + s_barrier below)
#pragma unroll
        for (int i = 0; i < PPW; ++i) {
            const unsigned dst = __builtin_amdgcn_readfirstlane(lds_base + buf_off + (wave + NW * i) * 1024);
            const T* src = gsrc[i] + (size_t)kt * GEMM_BK;
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep) : "v"(src), "s"(dst) : "memory");
        }
    };
#pragma unroll
    for (int i = 0; i < NSTAGE - 1; ++i) if (i < nk) stage(i, i * BUF_BYTES);
    int slot = 0;
    for (int kt = 0; kt < nk; ++kt) {
        const int rem = nk - 1 - kt;                         // tiles allowed to stay in flight past this wait: min(NSTAGE - 2, rem)
        if (NSTAGE >= 4 && rem >= 2) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(NSTAGE >= 4 ? 2 * PPW : 0) : "memory");
        else if (NSTAGE >= 3 && rem >= 1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(PPW) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();                        // tile kt visible to every wave; everyone is done reading the slot that is filled next
        if (kt + NSTAGE - 1 < nk) { int s2 = slot + NSTAGE - 1; s2 = s2 >= NSTAGE ? s2 - NSTAGE : s2; stage(kt + NSTAGE - 1, s2 * BUF_BYTES); }
        const char* buf = smem + slot * BUF_BYTES;
#pragma unroll
        for (int ks = 0; ks < GEMM_BK / 16; ++ks) {
            uint4 wf[NTL], xf[MT];
#pragma unroll
            for (int i = 0; i < NTL; ++i) wf[i] = *reinterpret_cast<const uint4*>(buf + lds_chunk_off(BM + wn * TN + i * 32 + l31, ks * 2 + hi));
#pragma unroll
            for (int j = 0; j < MT; ++j) xf[j] = *reinterpret_cast<const uint4*>(buf + lds_chunk_off(wm * TM + j * 32 + l31, ks * 2 + hi));
#pragma unroll
            for (int i = 0; i < NTL; ++i)
#pragma unroll
                for (int j = 0; j < MT; ++j) acc[i][j] = Mfma32x32x16<T>::run(wf[i], xf[j], acc[i][j]);
        }
        slot = slot + 1 == NSTAGE ? 0 : slot + 1;
    }
    const bool gated = act_gated(a.act);
#pragma unroll
    for (int j = 0; j < MT; ++j) {
        const int r = wm * TM + j * 32 + l31;
        if (r >= rows) continue;
        const int m = a.plan.order ? a.plan.order[row0 + r] : row0 + r;
        T* C = reinterpret_cast<T*>(a.C) + (size_t)m * a.ldc + (size_t)grp * a.c_group;
#pragma unroll
        for (int i = 0; i < NTL; ++i)
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int n = n0 + wn * TN + i * 32 + 8 * q + 4 * hi;      // (gated: 32 gate rows, then 32 up rows)
                if (n >= a.N || (gated && (i & 1))) continue;
                float v[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] = gated ? gate_mul(a.act, acc[i][j][4 * q + e], acc[i | 1][j][4 * q + e]) : acc[i][j][4 * q + e];
                store4<T>(C + (gated ? (n - 8 * q - 4 * hi) / 2 + 8 * q + 4 * hi : n), v);
            }
    }
}

template <typename T, int BM, int BN, int WM, int WN, int NSTAGE>
static void launch_group_gemm_cfg(const GroupGemmArgs& a, int m_tiles, hipStream_t st) {
    constexpr int smem = NSTAGE * (BM + BN) * GEMM_ROWB;
    static_assert(smem <= 160 * 1024, "LDS ring does not fit");
    auto kern = group_gemm_kernel<T, BM, BN, WM, WN, NSTAGE>;
    static bool attr_set = false;
    if (!attr_set) { LMX_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, smem)); attr_set = true; }
    LMX_LAUNCH(kern, dim3(m_tiles * cdiv(a.N, BN)), dim3(WM * WN * 64), smem, st, a);
    LMX_CHECK_HIP(hipGetLastError());
}
void launch_group_gemm(int dtype, const GroupGemmArgs& a, int bm, hipStream_t st) {
    LMX_REQUIRE(a.X && a.W && a.C && a.rows >= 1 && a.groups >= 1 && a.N >= 1 && a.K >= 64 && a.K % 64 == 0 && a.per_row >= 1, "group_gemm: bad arguments");
    LMX_REQUIRE(a.ldx % 8 == 0 && a.ldw % 8 == 0 && a.ldc % 4 == 0 && a.w_group % 8 == 0 && a.x_group % 8 == 0 && a.c_group % 4 == 0 && a.N % 4 == 0, "group_gemm: 16-byte rows");
    LMX_REQUIRE(!act_gated(a.act) || a.N % 64 == 0, "group_gemm: gated rows come in groups of 64");
    // with a plan: every group's last tile may be part empty; no more tiles than rows
    const int m_tiles = a.plan.n_tiles ? std::min(a.rows, a.rows / bm + a.groups) : a.groups * cdiv(a.rows, bm);
#define L(TT) do { if (bm == 32) launch_group_gemm_cfg<TT, 32, 128, 1, 2, 4>(a, m_tiles, st); else if (bm == 64) launch_group_gemm_cfg<TT, 64, 128, 2, 2, 3>(a, m_tiles, st); \
                   else if (bm == 128) launch_group_gemm_cfg<TT, 128, 128, 2, 2, 2>(a, m_tiles, st); else if (bm == 256) launch_group_gemm_cfg<TT, 256, 256, 2, 4, 2>(a, m_tiles, st); \
                   else throw Error{"group_gemm: tiles of 32, 64, 128 or 256 rows"}; } while (0)
    if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else throw Error{"group_gemm: 16-bit models"};
#undef L
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
