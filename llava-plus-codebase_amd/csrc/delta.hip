// Gated delta rule with a decay per key channel (kernels.h: DeltaShape).  Everything that enters the recurrence is fp32: unit norms, decays, step sizes, the state.
//
//   delta_prep_kernel    prompt rows: short convolutions and silu, unit q and k (and q . k), decays, step sizes -> scratch rows
//   delta_scan_kernel    prompt rows: the recurrence.  The columns of S (value channels) are independent of each other: DK / 8 lanes own one column, 8 key channels
//                        each in registers, so a wave walks 64 / (DK / 8) columns through the tokens; reductions are DPP adds inside the lane group
//   delta_gate_kernel    prompt rows: o / rms(o) * weight * sigmoid(gate)
//   delta_decode_kernel  one new token per sequence: all of it in one launch, one workgroup per head
//
// The read-out o = S^T q after the write equals (g S)^T q + (k . q) u, so both products of a token run over the decayed state at once and the state update is off the
// critical path.  The scan and the decode step use the same operation order per column.
#include "common.h"
#include "kernels.h"

namespace lmx {

// sum over the LPC lanes of a column (8, 16 or 32 consecutive lanes); every lane gets it
template <int CTRL> __device__ __forceinline__ float dpp_add(float v) {
    return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
template <int LPC> __device__ __forceinline__ float lanes_sum(float v) {
    v = dpp_add<0xB1>(v);                                  // lane ^ 1
    v = dpp_add<0x4E>(v);                                  // lane ^ 2
    v = dpp_add<0x141>(v);                                 // mirror in 8
    if constexpr (LPC >= 16) v = dpp_add<0x140>(v);        // mirror in 16
    if constexpr (LPC >= 32) v += __shfl_xor(v, 16, 64);
    return v;
}
__device__ __forceinline__ float softplus_f32(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float sigmoid_acc(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float decay_f32(float rate, float z) { return expf(-rate * softplus_f32(z)); }      // rate = exp(A_log)
__device__ __forceinline__ float silu_acc(float z) { return z / (1.f + expf(-z)); }

// ---------------------------------------------------------------------------------------------------------------
// prompt rows
// ---------------------------------------------------------------------------------------------------------------
constexpr int DELTA_TT = 32;             // tokens of one prep workgroup
constexpr int DELTA_TC = 16;             // tokens staged at a time by the scan

__device__ __forceinline__ const DeltaSeg* delta_segment(const DeltaPrefillArgs& a, int tile, int& t0) {
    for (int s = 0; s < a.n_seg; ++s) {
        const int nt = (a.seg[s].n + DELTA_TT - 1) / DELTA_TT;
        if (tile < nt) { t0 = tile * DELTA_TT; return &a.seg[s]; }
        tile -= nt;
    }
    return nullptr;
}

// 8 channels of token t: sum over the taps, then silu.  Inputs before the portion come from the ring, before the sequence they are zero
template <typename T>
__device__ __forceinline__ void conv_silu8(const DeltaPrefillArgs& a, const DeltaSeg& sg, int t, int c, float (&out)[8]) {
    const int taps = a.s.taps, C = a.s.channels();
    const T* w = reinterpret_cast<const T*>(a.w.conv) + c;
    const T* proj = reinterpret_cast<const T*>(a.proj) + (size_t)sg.row0 * a.ld + c;
    const T* ring = reinterpret_cast<const T*>(sg.ring) + c;
#pragma unroll
    for (int e = 0; e < 8; ++e) out[e] = 0.f;
    for (int j = 0; j < taps; ++j) {
        const int r = t - (taps - 1) + j, p = sg.pos0 + r;
        if (p < 0) continue;
        float x[8], f[8];
        load8<T>(r >= 0 ? proj + (size_t)r * a.ld : ring + (size_t)(p % taps) * C, x);
        load8<T>(w + (size_t)j * C, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) out[e] = fmaf(x[e], f[e], out[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) out[e] = silu_acc(out[e]);
}

template <typename T, int LPC>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrefillArgs a) {
    constexpr int DK = LPC * 8;
    const int tid = threadIdx.x, H = a.s.H, G = a.s.G, DV = a.s.DV;
    int t0 = 0;
    const DeltaSeg* sp = delta_segment(a, blockIdx.x, t0);
    if (!sp) return;
    const DeltaSeg sg = *sp;
    const int nt = sg.n - t0 < DELTA_TT ? sg.n - t0 : DELTA_TT;
    if ((int)blockIdx.y < G) {
        // one key head: q and k of a token by LPC lanes
        const int kh = blockIdx.y, sub = tid % LPC, rep = H / G;
        for (int t = t0 + tid / LPC; t < t0 + DELTA_TT; t += 256 / LPC) {      // every lane stays for the lane-group sums
            const bool live = t < t0 + nt;
            const int tt = live ? t : t0;
            float q[8], k[8];
            conv_silu8<T>(a, sg, tt, kh * DK + sub * 8, q);
            conv_silu8<T>(a, sg, tt, (G + kh) * DK + sub * 8, k);
            float qq = 0.f, kk = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) { qq = fmaf(q[e], q[e], qq); kk = fmaf(k[e], k[e], kk); }
            qq = lanes_sum<LPC>(qq); kk = lanes_sum<LPC>(kk);
            const float qi = 1.f / (sqrtf(qq + 1e-6f) * sqrtf((float)a.s.dk)), ki = 1.f / sqrtf(kk + 1e-6f);
            float kq = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) { q[e] *= qi; k[e] *= ki; kq = fmaf(q[e], k[e], kq); }
            kq = lanes_sum<LPC>(kq);
            if (!live) continue;
            const size_t row = (size_t)sg.row0 + t;
            float* o = a.qk + (row * G + kh) * 2 * DK + sub * 8;
            store8<float>(o, q); store8<float>(o + DK, k);
            for (int h = sub; h < rep; h += LPC) a.sc[(row * H + kh * rep + h) * 2 + 1] = kq;
        }
        return;
    }
    const int h = blockIdx.y - G;
    for (int i = tid; i < nt * (DV / 8); i += 256) {
        const int t = t0 + i / (DV / 8), c = (i % (DV / 8)) * 8;
        float v[8];
        conv_silu8<T>(a, sg, t, 2 * G * DK + h * DV + c, v);
        store8<T>(reinterpret_cast<T*>(a.v) + (((size_t)sg.row0 + t) * H + h) * DV + c, v);
    }
    const float rate = expf(to_f32(reinterpret_cast<const T*>(a.w.A_log)[h]));
    for (int i = tid; i < nt * LPC; i += 256) {
        const int c = (i % LPC) * 8;
        const size_t row = (size_t)sg.row0 + t0 + i / LPC;
        float z[8], d[8];
        load8<T>(reinterpret_cast<const T*>(a.ag) + row * a.ag_ld + h * DK + c, z);
        load8<T>(reinterpret_cast<const T*>(a.w.dt_bias) + h * DK + c, d);
#pragma unroll
        for (int e = 0; e < 8; ++e) z[e] = decay_f32(rate, z[e] + d[e]);
        store8<float>(a.g + (row * H + h) * DK + c, z);
    }
    for (int t = tid; t < nt; t += 256) {
        const size_t row = (size_t)sg.row0 + t0 + t;
        a.sc[(row * H + h) * 2] = sigmoid_acc(to_f32(reinterpret_cast<const T*>(a.proj)[row * a.ld + a.s.channels() + h]));
    }
}

template <typename T, int LPC>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaPrefillArgs a) {
    constexpr int DK = LPC * 8, CPW = 64 / LPC, CPB = 4 * CPW, TC = DELTA_TC;
    __shared__ __attribute__((aligned(16))) float kqg[TC][3][DK];
    __shared__ float vs[TC][CPB], os[TC][CPB];
    __shared__ float2 sc[TC];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int H = a.s.H, G = a.s.G, DV = a.s.DV;
    const int nblk = DV / CPB, h = blockIdx.x / nblk, c0 = (blockIdx.x % nblk) * CPB, kh = h / (H / G);
    const DeltaSeg sg = a.seg[blockIdx.y];
    const int sub = lane % LPC, col = wave * CPW + lane / LPC;
    float* st = sg.state + ((size_t)h * DV + c0 + col) * DK + sub * 8;
    float S[8];
    if (sg.pos0 > 0) load8<float>(st, S);
    else {
#pragma unroll
        for (int e = 0; e < 8; ++e) S[e] = 0.f;
    }
    // a chunk's rows: global -> registers while the chunk before is walked -> LDS
    constexpr int NQ = TC * DK / 4, QPT = NQ / 256;          // float4s of one of k, q, g per thread
    static_assert(NQ % 256 == 0, "whole passes");
    float4 rk[QPT], rq[QPT], rg[QPT];
    float rv[(TC * CPB + 255) / 256];
    float2 rs;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < QPT; ++i) {
            const int f = tid + i * 256, t = f / (DK / 4), c = (f % (DK / 4)) * 4;
            const size_t row = (size_t)sg.row0 + (t0 + t < sg.n ? t0 + t : sg.n - 1);
            const float* qp = a.qk + (row * G + kh) * 2 * DK + c;
            rq[i] = *reinterpret_cast<const float4*>(qp); rk[i] = *reinterpret_cast<const float4*>(qp + DK);
            rg[i] = *reinterpret_cast<const float4*>(a.g + (row * H + h) * DK + c);
        }
#pragma unroll
        for (int i = 0; i < (TC * CPB + 255) / 256; ++i) {
            const int f = tid + i * 256, t = f / CPB;
            const size_t row = (size_t)sg.row0 + (t0 + t < sg.n ? t0 + t : sg.n - 1);
            if (f < TC * CPB) rv[i] = to_f32(reinterpret_cast<const T*>(a.v)[(row * H + h) * DV + c0 + f % CPB]);
        }
        if (tid < TC) {
            const size_t row = (size_t)sg.row0 + (t0 + tid < sg.n ? t0 + tid : sg.n - 1);
            rs = *reinterpret_cast<const float2*>(a.sc + (row * H + h) * 2);
        }
    };
    auto put = [&]() {
#pragma unroll
        for (int i = 0; i < QPT; ++i) {
            const int f = tid + i * 256, t = f / (DK / 4), c = (f % (DK / 4)) * 4;
            *reinterpret_cast<float4*>(&kqg[t][0][c]) = rk[i]; *reinterpret_cast<float4*>(&kqg[t][1][c]) = rq[i]; *reinterpret_cast<float4*>(&kqg[t][2][c]) = rg[i];
        }
#pragma unroll
        for (int i = 0; i < (TC * CPB + 255) / 256; ++i) { const int f = tid + i * 256; if (f < TC * CPB) vs[f / CPB][f % CPB] = rv[i]; }
        if (tid < TC) sc[tid] = rs;
    };
    fetch(0);
    for (int t0 = 0; t0 < sg.n; t0 += TC) {
        put();
        __syncthreads();
        if (t0 + TC < sg.n) fetch(t0 + TC);
        const int nt = sg.n - t0 < TC ? sg.n - t0 : TC;
        for (int t = 0; t < nt; ++t) {
            float k[8], q[8], g[8];
            load8<float>(&kqg[t][0][sub * 8], k); load8<float>(&kqg[t][1][sub * 8], q); load8<float>(&kqg[t][2][sub * 8], g);
            const float2 bk = sc[t];
            float r0 = 0.f, r1 = 0.f, o0 = 0.f, o1 = 0.f;
#pragma unroll
            for (int e = 0; e < 8; e += 2) {
                S[e] *= g[e]; S[e + 1] *= g[e + 1];
                r0 = fmaf(S[e], k[e], r0); r1 = fmaf(S[e + 1], k[e + 1], r1);
                o0 = fmaf(S[e], q[e], o0); o1 = fmaf(S[e + 1], q[e + 1], o1);
            }
            const float r = lanes_sum<LPC>(r0 + r1), o = lanes_sum<LPC>(o0 + o1);
            const float u = bk.x * (vs[t][col] - r);
#pragma unroll
            for (int e = 0; e < 8; ++e) S[e] = fmaf(k[e], u, S[e]);
            if (sub == 0) os[t][col] = fmaf(bk.y, u, o);
        }
        __syncthreads();
        for (int f = tid; f < nt * CPB; f += 256) a.o[(((size_t)sg.row0 + t0 + f / CPB) * H + h) * DV + c0 + f % CPB] = os[f / CPB][f % CPB];
    }
    store8<float>(st, S);
    // the newest inputs of the convolutions: every channel once, spread over the segment's workgroups
    const int C = a.s.channels(), taps = a.s.taps, keep = sg.n < taps ? sg.n : taps;
    for (int c = blockIdx.x * 256 + tid; c < C; c += gridDim.x * 256)
        for (int j = 0; j < keep; ++j) {
            const int t = sg.n - keep + j;
            reinterpret_cast<T*>(sg.ring)[(size_t)((sg.pos0 + t) % taps) * C + c] = reinterpret_cast<const T*>(a.proj)[((size_t)sg.row0 + t) * a.ld + c];
        }
}

// one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_gate_kernel(DeltaPrefillArgs a, int pairs, int row_base) {
    const int lane = threadIdx.x & 63, p = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (p >= pairs) return;
    const int H = a.s.H, DV = a.s.DV, h = p % H;
    const size_t row = (size_t)row_base + p / H;
    const float* o = a.o + (row * H + h) * DV;
    float ss = 0.f;
    for (int c = lane; c < DV; c += 64) ss += o[c] * o[c];
    const float inv = 1.f / sqrtf(wave_sum(ss) / (float)a.s.dv + a.eps);
    const T* gate = reinterpret_cast<const T*>(a.ag) + row * a.ag_ld + H * a.s.DK + h * DV;
    const T* w = reinterpret_cast<const T*>(a.w.norm);
    T* out = reinterpret_cast<T*>(a.out) + row * a.out_ld + h * DV;
    for (int c = lane; c < DV; c += 64) out[c] = from_f32<T>(o[c] * inv * to_f32(w[c]) * sigmoid_acc(to_f32(gate[c])));
}

size_t delta_scratch_bytes(const DeltaShape& s, int rows, int es) {
    auto up = [](size_t b) { return (b + 255) / 256 * 256; };
    const size_t r = (size_t)rows;
    return up(r * s.G * 2 * s.DK * 4) + up(r * s.H * s.DK * 4) + up(r * s.H * s.DV * es) + up(r * s.H * 8) + up(r * s.H * s.DV * 4);
}
void delta_carve(DeltaPrefillArgs& a, void* scratch, int rows, int es) {
    auto up = [](size_t b) { return (b + 255) / 256 * 256; };
    char* p = static_cast<char*>(scratch);
    const size_t r = (size_t)rows;
    a.qk = reinterpret_cast<float*>(p); p += up(r * a.s.G * 2 * a.s.DK * 4);
    a.g = reinterpret_cast<float*>(p); p += up(r * a.s.H * a.s.DK * 4);
    a.v = p; p += up(r * a.s.H * a.s.DV * es);
    a.sc = reinterpret_cast<float*>(p); p += up(r * a.s.H * 8);
    a.o = reinterpret_cast<float*>(p);
}

static void delta_check(const DeltaShape& s) {
    LMX_REQUIRE(s.H >= 1 && s.G >= 1 && s.H % s.G == 0, "delta: heads must be a multiple of key heads");
    LMX_REQUIRE((s.DK == 64 || s.DK == 128 || s.DK == 256) && s.DV >= 64 && s.DV % 64 == 0 && s.dk >= 1 && s.dk <= s.DK && s.dv >= 1 && s.dv <= s.DV, "delta: bad head widths");
    LMX_REQUIRE(s.taps >= 1, "delta: at least one tap");
}
static void delta_check(const DeltaPrefillArgs& a) {
    delta_check(a.s);
    LMX_REQUIRE(a.ld % 8 == 0 && a.ld >= a.s.channels() + a.s.H && a.ag_ld % 8 == 0 && a.ag_ld >= a.s.H * (a.s.DK + a.s.DV), "delta: bad row pitch");
    LMX_REQUIRE(a.n_seg >= 1 && a.n_seg <= DELTA_MAX_SEG, "delta: 1..16 segments a launch");
    for (int i = 0; i < a.n_seg; ++i) LMX_REQUIRE(a.seg[i].n >= 1 && a.seg[i].pos0 >= 0 && a.seg[i].row0 >= 0 && a.seg[i].state && a.seg[i].ring, "delta: bad segment");
}
#define DELTA_K(KERN, GRID, SMEM, ...) do { if (a.s.DK == 64) LMX_LAUNCH((KERN<TT, 8>), GRID, dim3(256), SMEM, st, __VA_ARGS__); \
                                            else if (a.s.DK == 128) LMX_LAUNCH((KERN<TT, 16>), GRID, dim3(256), SMEM, st, __VA_ARGS__); \
                                            else LMX_LAUNCH((KERN<TT, 32>), GRID, dim3(256), SMEM, st, __VA_ARGS__); } while (0)

void launch_delta_prep(int dtype, const DeltaPrefillArgs& a, hipStream_t st) {
    delta_check(a);
    int tiles = 0;
    for (int i = 0; i < a.n_seg; ++i) tiles += cdiv(a.seg[i].n, DELTA_TT);
    const dim3 grid(tiles, a.s.G + a.s.H);
    if (dtype == kBF16) { using TT = bf16_t; DELTA_K(delta_prep_kernel, grid, 0, a); }
    else if (dtype == kF16) { using TT = f16_t; DELTA_K(delta_prep_kernel, grid, 0, a); }
    else { using TT = float; DELTA_K(delta_prep_kernel, grid, 0, a); }
    LMX_CHECK_HIP(hipGetLastError());
}
void launch_delta_scan(int dtype, const DeltaPrefillArgs& a, hipStream_t st) {
    delta_check(a);
    const int cpb = 4 * 64 / (a.s.DK / 8);
    const dim3 grid(a.s.H * (a.s.DV / cpb), a.n_seg);
    if (dtype == kBF16) { using TT = bf16_t; DELTA_K(delta_scan_kernel, grid, 0, a); }
    else if (dtype == kF16) { using TT = f16_t; DELTA_K(delta_scan_kernel, grid, 0, a); }
    else { using TT = float; DELTA_K(delta_scan_kernel, grid, 0, a); }
    LMX_CHECK_HIP(hipGetLastError());
}
void launch_delta_gate(int dtype, const DeltaPrefillArgs& a, hipStream_t st) {
    delta_check(a);
    for (int i = 0; i < a.n_seg;) {                          // neighbouring segments are one run of rows
        int k = i + 1, rows = a.seg[i].n;
        while (k < a.n_seg && a.seg[k].row0 == a.seg[k - 1].row0 + a.seg[k - 1].n) rows += a.seg[k++].n;
        const int pairs = rows * a.s.H;
#define L(TT) LMX_LAUNCH(delta_gate_kernel<TT>, dim3(cdiv(pairs, 4)), dim3(256), 0, st, a, pairs, a.seg[i].row0)
        if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
        i = k;
    }
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// one new token per sequence: grid (heads, sequences), 256 threads
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int LPC>
__global__ __launch_bounds__(256) void delta_decode_kernel(DeltaDecodeArgs a) {
    constexpr int DK = LPC * 8, CPP = 256 / LPC;             // columns of one pass over the state
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int H = a.s.H, G = a.s.G, DV = a.s.DV, taps = a.s.taps, C = a.s.channels();
    const int h = blockIdx.x, z = blockIdx.y, rep = H / G, kh = h / rep;
    float *q = sm, *k = q + DK, *g = k + DK, *v = g + DK, *gate = v + DV, *o = gate + DV, *lat = o + DV;      // lat [ra + rg]
    __shared__ float red[4], kq_s;
    const DecodeFusedSeq e = a.tab ? a.tab[z] : a.one;
    const int pos = *e.pos_ptr;
    const bool frozen = e.done && *e.done != 0;
    const T* row = reinterpret_cast<const T*>(a.proj) + (size_t)z * a.ld;
    float* st = reinterpret_cast<float*>(e.K) + (size_t)h * DV * DK;
    T* ring = reinterpret_cast<T*>(e.VT);
    const T* conv = reinterpret_cast<const T*>(a.w.conv);
    const int sub = tid % LPC, col = tid / LPC;
    // the first passes over the state are requested before anything waits
    constexpr int PF = 4;
    float S[PF][8];
#pragma unroll
    for (int p = 0; p < PF; ++p) if (p * CPP + col < DV) load8<float>(st + (size_t)(p * CPP + col) * DK + sub * 8, S[p]);
    // ---- short convolutions: thread per channel; the ring slot of this position is not one that any tap reads
    for (int i = tid; i < 2 * DK + DV; i += 256) {
        const bool is_v = i >= 2 * DK;
        const int c = is_v ? 2 * G * DK + h * DV + i - 2 * DK : (i < DK ? kh * DK + i : (G + kh) * DK + i - DK);
        const T xin = row[c];
        float s = to_f32(xin) * to_f32(conv[(size_t)(taps - 1) * C + c]);
        for (int j = 1; j < taps; ++j) if (pos - j >= 0) s = fmaf(to_f32(ring[(size_t)((pos - j) % taps) * C + c]), to_f32(conv[(size_t)(taps - 1 - j) * C + c]), s);
        if (is_v || h % rep == 0) ring[(size_t)(pos % taps) * C + c] = xin;
        s = silu_acc(s);
        if (is_v) v[i - 2 * DK] = s; else sm[i] = s;
    }
    for (int i = tid; i < a.ra + a.rg; i += 256) lat[i] = to_f32(row[a.a_off + i]);
    __syncthreads();
    if (wave < 2) {
        float* x = wave == 0 ? q : k;
        float ss = 0.f;
        for (int i = lane; i < DK; i += 64) ss += x[i] * x[i];
        float inv = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
        if (wave == 0) inv *= 1.f / sqrtf((float)a.s.dk);
        for (int i = lane; i < DK; i += 64) x[i] *= inv;
    }
    // ---- decays and output gates: 8 lanes per row of the second low-rank matrices
    const float rate = expf(to_f32(reinterpret_cast<const T*>(a.w.A_log)[h]));
    for (int i = tid >> 3; i < DK + DV; i += 32) {
        const bool is_g = i < DK;
        const T* w = reinterpret_cast<const T*>(a.wag) + (size_t)(is_g ? h * DK + i : H * DK + h * DV + i - DK) * a.wag_ld + (is_g ? 0 : a.ra);
        const float* x = is_g ? lat : lat + a.ra;
        float s = 0.f;
        for (int c = (tid & 7) * 8; c < (is_g ? a.ra : a.rg); c += 64) {
            float f[8]; load8<T>(w + c, f);
#pragma unroll
            for (int n = 0; n < 8; ++n) s = fmaf(f[n], x[c + n], s);
        }
        s = lanes_sum<8>(s);
        s = round_to<T>(s);                                  // the prompt path stores this product in the model dtype
        if ((tid & 7) == 0) {
            if (is_g) g[i] = decay_f32(rate, s + to_f32(reinterpret_cast<const T*>(a.w.dt_bias)[h * DK + i]));
            else gate[i - DK] = sigmoid_acc(s);
        }
    }
    __syncthreads();
    if (wave == 0) {
        float s = 0.f;
        for (int i = lane; i < DK; i += 64) s = fmaf(q[i], k[i], s);
        s = wave_sum(s);
        if (lane == 0) kq_s = s;
    }
    __syncthreads();
    const float beta = sigmoid_acc(to_f32(row[C + h])), kq = kq_s;
    float kr[8], qr[8], gr[8];
    load8<float>(k + sub * 8, kr); load8<float>(q + sub * 8, qr); load8<float>(g + sub * 8, gr);
    float ss = 0.f;
    auto column = [&](float (&s)[8], int c) {
        float r0 = 0.f, r1 = 0.f, o0 = 0.f, o1 = 0.f;
#pragma unroll
        for (int n = 0; n < 8; n += 2) {
            s[n] *= gr[n]; s[n + 1] *= gr[n + 1];
            r0 = fmaf(s[n], kr[n], r0); r1 = fmaf(s[n + 1], kr[n + 1], r1);
            o0 = fmaf(s[n], qr[n], o0); o1 = fmaf(s[n + 1], qr[n + 1], o1);
        }
        const float r = lanes_sum<LPC>(r0 + r1), oo = lanes_sum<LPC>(o0 + o1);
        const float u = beta * (round_to<T>(v[c]) - r);
#pragma unroll
        for (int n = 0; n < 8; ++n) s[n] = fmaf(kr[n], u, s[n]);
        const float out = fmaf(kq, u, oo);
        if (sub == 0) { o[c] = out; ss += out * out; }
        if (!frozen) store8<float>(st + (size_t)c * DK + sub * 8, s);
    };
    for (int c0 = 0; c0 < DV; c0 += PF * CPP) {
#pragma unroll
        for (int p = 0; p < PF; ++p) {
            const int c = c0 + p * CPP + col;
            if (c < DV) column(S[p], c);                     // uniform in a lane group
        }
#pragma unroll
        for (int p = 0; p < PF; ++p) {
            const int c = c0 + (PF + p) * CPP + col;
            if (c < DV) load8<float>(st + (size_t)c * DK + sub * 8, S[p]);
        }
    }
    ss = block_sum<4>(ss, red);                              // (its barriers also publish o)
    const float inv = 1.f / sqrtf(ss / (float)a.s.dv + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)z * a.out_ld + h * DV;
    for (int c = tid; c < DV; c += 256) out[c] = from_f32<T>(o[c] * inv * to_f32(reinterpret_cast<const T*>(a.w.norm)[c]) * gate[c]);
}

void launch_delta_decode(int dtype, const DeltaDecodeArgs& a, hipStream_t st) {
    delta_check(a.s);
    LMX_REQUIRE(a.ra % 64 == 0 && a.rg % 64 == 0 && a.ra >= 64 && a.rg >= 64 && a.wag_ld >= a.ra + a.rg && a.wag_ld % 8 == 0, "delta_decode: low-rank widths in whole 64-column groups");
    LMX_REQUIRE(a.a_off >= a.s.channels() + a.s.H && a.ld >= a.a_off + a.ra + a.rg, "delta_decode: bad row pitch");
    LMX_REQUIRE(a.n_seq >= 1 && (a.tab || (a.n_seq == 1 && a.one.K && a.one.VT && a.one.pos_ptr)), "delta_decode: bad sequence");
    const dim3 grid(a.s.H, a.n_seq);
    const size_t smem = (size_t)(3 * a.s.DK + 3 * a.s.DV + a.ra + a.rg) * 4;
    LMX_REQUIRE(smem <= 64 * 1024, "delta_decode: low-rank widths too large");
    if (dtype == kBF16) { using TT = bf16_t; DELTA_K(delta_decode_kernel, grid, smem, a); }
    else if (dtype == kF16) { using TT = f16_t; DELTA_K(delta_decode_kernel, grid, smem, a); }
    else { using TT = float; DELTA_K(delta_decode_kernel, grid, smem, a); }
    LMX_CHECK_HIP(hipGetLastError());
}

}  // namespace lmx
