// Gated delta rule with a decay per key channel (kernels.h: DeltaShape).  Everything that enters the recurrence is fp32: unit norms, decays, step sizes, the state.
//
//   delta_prep_kernel    prompt rows: short convolutions and silu, unit q and k, decays, step sizes, and per chunk of 16 tokens what the recurrence needs of them
//   delta_scan_kernel    prompt rows: the recurrence, chunk by chunk, on fp32 MFMA tiles; a workgroup owns 16 columns of S (value channels), its 4 waves the key channels
//   delta_gate_kernel    prompt rows: o / rms(o) * weight * sigmoid(gate)
//   delta_decode_kernel  one new token per sequence: all of it in one launch, one workgroup per head
//
// A chunk.  With D_t the product of the chunk's decays up to token t (elementwise over key channels) and S the state before the chunk, the recurrence unrolls to
//   u_t = beta_t (v_t - (D_t k_t)^T S - sum_{s<t} A_ts u_s)      A_ts = k_t . (D_t / D_s) k_s
//   o_t = (D_t q_t)^T S + sum_{s<=t} P_ts u_s                    P_ts = q_t . (D_t / D_s) k_s
//   S'  = D_15 S + sum_s ((D_15 / D_s) k_s) u_s^T
// The quotients are products of the decays in between, never divisions, so a decay of any strength is exact to rounding.  A, P and T = (1 + diag(beta) A)^-1 diag(beta)
// (unit lower triangular: forward substitution) do not depend on S: delta_prep_kernel forms them for all chunks at once, the scan is left with U = T (V - (D k) S) and
// the products above.
//
// Decode: the read-out o = S^T q after the write equals (g S)^T q + (k . q) u, so both products of a token run over the decayed state at once and the state update is
// off the critical path.
#include <algorithm>
#include <type_traits>

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
constexpr int DELTA_C = 16;              // tokens of a chunk

// segment of a chunk (its index, or -1)
__device__ __forceinline__ int delta_segment(const DeltaPrefillArgs& a, int chunk) {
    int s = a.n_seg - 1;
    while (s > 0 && a.seg[s].chunk0 > chunk) --s;
    return (chunk - a.seg[s].chunk0) * DELTA_C < a.seg[s].n ? s : -1;
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
#pragma unroll 4
    for (int j = 0; j < taps; ++j) {
        const int r = t - (taps - 1) + j, p = sg.pos0 + r;
        if (p < 0) continue;
        float x[8], f[8];
        const T* src = proj + (ptrdiff_t)r * a.ld;
        if (r < 0) src = ring + (size_t)(p % taps) * C;
        load8<T>(src, x);
        load8<T>(w + (size_t)j * C, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) out[e] = fmaf(x[e], f[e], out[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) out[e] = silu_acc(out[e]);
}

// grid (chunks, heads), 256 threads
template <typename T, int LPC>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrefillArgs a) {
    constexpr int DK = LPC * 8, C = DELTA_C, CW = DK / 16;
    extern __shared__ __attribute__((aligned(16))) float dsm[];
    float *g = dsm, *k = g + C * DK, *q = k + C * DK;        // [C][DK]; the value tile comes first in the same place, the written-out keys last
    __shared__ float A[C][C], P[C][C], beta[C];
    const int tid = threadIdx.x, H = a.s.H, G = a.s.G, DV = a.s.DV;
    const int si = __builtin_amdgcn_readfirstlane(delta_segment(a, blockIdx.x));
    if (si < 0) return;
    const DeltaSeg sg = a.seg[si];
    const int t0 = ((int)blockIdx.x - sg.chunk0) * DELTA_C;
    const int nt = sg.n - t0 < C ? sg.n - t0 : C;
    const int h = blockIdx.y, kh = h / (H / G);
    const size_t ch = (size_t)(sg.chunk0 + t0 / C) * H + h;
    // ---- values, transposed: [DV][C]
    T* vt = reinterpret_cast<T*>(dsm);
    for (int i = tid; i < C * (DV / 8); i += 256) {
        const int t = i / (DV / 8), c = (i % (DV / 8)) * 8;
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = 0.f;
        if (t < nt) conv_silu8<T>(a, sg, t0 + t, 2 * G * DK + h * DV + c, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) vt[(c + e) * C + t] = from_f32<T>(v[e]);
    }
    __syncthreads();
    {
        const uint4* src = reinterpret_cast<const uint4*>(dsm);
        uint4* dst = reinterpret_cast<uint4*>(reinterpret_cast<T*>(a.v) + ch * DV * C);
        for (int i = tid; i < DV * C * (int)sizeof(T) / 16; i += 256) dst[i] = src[i];
    }
    __syncthreads();
    // ---- unit q and k (rows 0..15: q, 16..31: k); tokens past the portion are zero rows with decay 1
    for (int r = tid / LPC; r < 2 * C; r += 256 / LPC) {
        const int t = r % C, c = (tid % LPC) * 8;
        const bool is_k = r >= C;
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = 0.f;
        if (t < nt) conv_silu8<T>(a, sg, t0 + t, (is_k ? G + kh : kh) * DK + c, x);
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf(x[e], x[e], ss);
        ss = lanes_sum<LPC>(ss);
        const float inv = is_k ? 1.f / sqrtf(ss + 1e-6f) : 1.f / (sqrtf(ss + 1e-6f) * sqrtf((float)a.s.dk));
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= inv;
        store8<float>((is_k ? k : q) + t * DK + c, x);
    }
    const float rate = expf(to_f32(reinterpret_cast<const T*>(a.w.A_log)[h]));
    for (int i = tid; i < C * LPC; i += 256) {
        const int t = i / LPC, c = (i % LPC) * 8;
        float z[8], d[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) z[e] = 1.f;
        if (t < nt) {
            load8<T>(reinterpret_cast<const T*>(a.ag) + ((size_t)sg.row0 + t0 + t) * a.ag_ld + h * DK + c, z);
            load8<T>(reinterpret_cast<const T*>(a.w.dt_bias) + h * DK + c, d);
#pragma unroll
            for (int e = 0; e < 8; ++e) z[e] = decay_f32(rate, z[e] + d[e]);
        }
        store8<float>(g + t * DK + c, z);
    }
    if (tid < C) beta[tid] = tid < nt ? sigmoid_acc(to_f32(reinterpret_cast<const T*>(a.proj)[((size_t)sg.row0 + t0 + tid) * a.ld + a.s.channels() + h])) : 0.f;
    A[tid / C][tid % C] = 0.f; P[tid / C][tid % C] = 0.f;
    __syncthreads();
    // ---- A and P: 16 lanes own one key s and carry it through the decays behind it
    const int s = tid / 16, sub = tid % 16;
    float r[CW];
#pragma unroll
    for (int j = 0; j < CW / 4; ++j) {
        const float4 x = *reinterpret_cast<const float4*>(k + s * DK + j * 64 + sub * 4);
        r[j * 4] = x.x; r[j * 4 + 1] = x.y; r[j * 4 + 2] = x.z; r[j * 4 + 3] = x.w;
    }
    for (int t = (tid >> 6) * 4; t < C; ++t) {
        float ak = 0.f, aq = 0.f;
#pragma unroll
        for (int j = 0; j < CW / 4; ++j) {
            const int c = t * DK + j * 64 + sub * 4;
            const float4 gg = *reinterpret_cast<const float4*>(g + c), kk = *reinterpret_cast<const float4*>(k + c), qq = *reinterpret_cast<const float4*>(q + c);
            if (t > s) { r[j * 4] *= gg.x; r[j * 4 + 1] *= gg.y; r[j * 4 + 2] *= gg.z; r[j * 4 + 3] *= gg.w; }
            ak = fmaf(kk.x, r[j * 4], ak); ak = fmaf(kk.y, r[j * 4 + 1], ak); ak = fmaf(kk.z, r[j * 4 + 2], ak); ak = fmaf(kk.w, r[j * 4 + 3], ak);
            aq = fmaf(qq.x, r[j * 4], aq); aq = fmaf(qq.y, r[j * 4 + 1], aq); aq = fmaf(qq.z, r[j * 4 + 2], aq); aq = fmaf(qq.w, r[j * 4 + 3], aq);
        }
        ak = lanes_sum<16>(ak); aq = lanes_sum<16>(aq);
        if (sub == 0 && t >= s) { P[t][s] = aq; if (t > s) A[t][s] = ak; }
    }
    // ---- D_t k_t, D_t q_t, D_15
    {
        constexpr int PARTS = 256 / DK;
        const int c = tid % DK, part = tid / DK;
        float D = 1.f;
#pragma unroll
        for (int t = 0; t < C; ++t) {
            D *= g[t * DK + c];
            if (t % PARTS != part) continue;
            a.kd[(ch * C + t) * DK + c] = D * k[t * DK + c];
            a.qd[(ch * C + t) * DK + c] = D * q[t * DK + c];
        }
        if (part == 0) a.dc[ch * DK + c] = D;
    }
    __syncthreads();
    a.pm[ch * C * C + tid] = P[tid / C][tid % C];
    if (tid < C) {                                           // column tid of T
        float x[C];
#pragma unroll
        for (int t = 0; t < C; ++t) {
            float v = t == tid ? 1.f : 0.f;
#pragma unroll
            for (int i = 0; i < t; ++i) v = fmaf(-A[t][i], x[i], v);
            x[t] = beta[t] * v;
            a.tm[(ch * C + t) * C + tid] = x[t];
        }
    }
#pragma unroll
    for (int j = 0; j < CW; ++j) dsm[((j / 4) * 64 + sub * 4 + j % 4) * (C + 1) + s] = r[j];
    __syncthreads();
    for (int i = tid; i < DK * C; i += 256) a.kt[ch * DK * C + i] = dsm[(i / C) * (C + 1) + i % C];
}

__device__ __forceinline__ f32x4 mfma4(float a, float b, const f32x4& c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ f32x4 ldg4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }

// grid (heads x DV / 16, segments), 256 threads: wave w owns key channels [w DK / 4, (w + 1) DK / 4) of 16 columns.  Everything is laid out so that no operand changes
// lanes: register i of lane l of an accumulator is row 4 (l / 16) + i, column l % 16, which as a B operand is k index l / 16 of the i-th of four products whose A operands
// hold columns 4 (l / 16) + i.  The waves' parts of (D k) S and of o meet in LDS.
template <typename T, int LPC>
__global__ __launch_bounds__(256, 1) void delta_scan_kernel(DeltaPrefillArgs a) {
    constexpr int DK = LPC * 8, NT = DK / 64, C = DELTA_C;
    __shared__ __attribute__((aligned(16))) f32x4 wb[2][4][64], ob[2][4][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int H = a.s.H, DV = a.s.DV;
    const int lid = xcd_remap(blockIdx.x, gridDim.x), nblk = DV / 16, h = lid / nblk, c0 = (lid % nblk) * 16;
    const DeltaSeg sg = a.seg[blockIdx.y];
    const int r16 = lane & 15, q4 = (lane >> 4) * 4, cb = wave * (DK / 4);
    float* st = sg.state + ((size_t)h * DV + c0 + r16) * DK + cb + q4;
    f32x4 S[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) S[j] = sg.pos0 > 0 ? ldg4(st + j * 16) : f32x4{0.f, 0.f, 0.f, 0.f};
    using Raw = std::conditional_t<sizeof(T) == 2, uint2, f32x4>;
    struct Chunk { f32x4 kd[NT], qd[NT], kt[NT], dc[NT], tm; float pm; Raw v; };
    auto fetch = [&](int n, Chunk& x) {
        const size_t ch = (size_t)(sg.chunk0 + n) * H + h;
#pragma unroll
        for (int j = 0; j < NT; ++j) {
            const int c = cb + j * 16;
            x.kd[j] = ldg4(a.kd + (ch * C + r16) * DK + c + q4);
            x.qd[j] = ldg4(a.qd + (ch * C + r16) * DK + c + q4);
            x.kt[j] = ldg4(a.kt + (ch * DK + c + r16) * C + q4);
            x.dc[j] = ldg4(a.dc + ch * DK + c + q4);
        }
        x.tm = ldg4(a.tm + (ch * C + r16) * C + q4);
        x.pm = a.pm[(ch * C + r16) * C + q4 + wave];
        x.v = *reinterpret_cast<const Raw*>(reinterpret_cast<const T*>(a.v) + (ch * DV + c0 + r16) * C + q4);
    };
    auto put_o = [&](int n) {                                // chunk n's read-out, one element a thread
        const int t = ((tid >> 2) >> 4) * 4 + (tid & 3), col = (tid >> 2) & 15;
        const float* p = reinterpret_cast<const float*>(&ob[n & 1][0][0]) + tid;
        const float v = (p[0] + p[256]) + (p[512] + p[768]);
        if (n * C + t < sg.n) a.o[((size_t)sg.row0 + n * C + t) * H * DV + (size_t)h * DV + c0 + col] = v;
    };
    const int nc = (sg.n + C - 1) / C;
    auto step = [&](int n, const Chunk& cur) {
        f32x4 W = {0.f, 0.f, 0.f, 0.f}, O = W, U = W, X;
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) W = mfma4(cur.kd[j][i], S[j][i], W);
        wb[n & 1][wave][lane] = W;
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = mfma4(cur.qd[j][i], S[j][i], O);
        // LDS only: a full barrier would also wait for the chunks that are on their way
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        const f32x4 w0 = wb[n & 1][0][lane], w1 = wb[n & 1][1][lane], w2 = wb[n & 1][2][lane], w3 = wb[n & 1][3][lane];
        f32x4 v;
        if constexpr (sizeof(T) == 2) v = f32x4{unpack_lo<T>(cur.v.x), unpack_hi<T>(cur.v.x), unpack_lo<T>(cur.v.y), unpack_hi<T>(cur.v.y)}; else v = cur.v;
#pragma unroll
        for (int i = 0; i < 4; ++i) X[i] = v[i] - ((w0[i] + w1[i]) + (w2[i] + w3[i]));
#pragma unroll
        for (int i = 0; i < 4; ++i) U = mfma4(cur.tm[i], X[i], U);
#pragma unroll
        for (int j = 0; j < NT; ++j) {
#pragma unroll
            for (int i = 0; i < 4; ++i) S[j][i] *= cur.dc[j][i];
#pragma unroll
            for (int i = 0; i < 4; ++i) S[j] = mfma4(cur.kt[j][i], U[i], S[j]);
        }
        O = mfma4(cur.pm, wave == 0 ? U[0] : wave == 1 ? U[1] : wave == 2 ? U[2] : U[3], O);      // a quarter of P U per wave
        ob[n & 1][wave][lane] = O;
        if (n > 0) put_o(n - 1);
    };
    // NB chunks in registers, NB - 1 of them on their way; past the last chunk the last one is read again
    constexpr int NB = NT >= 4 ? 3 : 4;
    Chunk buf[NB];
    auto at = [&](int n) { return n < nc ? n : nc - 1; };
#pragma unroll
    for (int u = 0; u < NB - 1; ++u) fetch(at(u), buf[u]);
    int n = 0;
    for (; n + NB <= nc; n += NB)
#pragma unroll
        for (int u = 0; u < NB; ++u) { fetch(at(n + u + NB - 1), buf[(u + NB - 1) % NB]); step(n + u, buf[u]); }
#pragma unroll
    for (int u = 0; u < NB - 1; ++u) if (n + u < nc) step(n + u, buf[u]);
    __syncthreads();
    put_o(nc - 1);
#pragma unroll
    for (int j = 0; j < NT; ++j) *reinterpret_cast<f32x4*>(st + j * 16) = S[j];
    // the newest inputs of the convolutions: every channel once, spread over the segment's workgroups
    const int CH = a.s.channels(), taps = a.s.taps, keep = sg.n < taps ? sg.n : taps;
    for (int c = blockIdx.x * 256 + tid; c < CH; c += gridDim.x * 256)
        for (int j = 0; j < keep; ++j) {
            const int t = sg.n - keep + j;
            reinterpret_cast<T*>(sg.ring)[(size_t)((sg.pos0 + t) % taps) * CH + c] = reinterpret_cast<const T*>(a.proj)[((size_t)sg.row0 + t) * a.ld + c];
        }
}

// `lpv` lanes (a power of two, 8 lpv >= DV) per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_gate_kernel(DeltaPrefillArgs a, int pairs, int row_base, int lpv) {
    const int p = blockIdx.x * (256 / lpv) + threadIdx.x / lpv, c = (threadIdx.x % lpv) * 8, pp = p < pairs ? p : pairs - 1;      // every lane stays for the sums
    const int H = a.s.H, DV = a.s.DV, h = pp % H, cc = c < DV ? c : 0;
    const size_t row = (size_t)row_base + pp / H;
    float o[8], gate[8], w[8], ss = 0.f;
    load8<float>(a.o + (row * H + h) * DV + cc, o);
    load8<T>(reinterpret_cast<const T*>(a.ag) + row * a.ag_ld + H * a.s.DK + h * DV + cc, gate);
    load8<T>(reinterpret_cast<const T*>(a.w.norm) + cc, w);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = fmaf(o[e], o[e], ss);
    ss = c < DV ? ss : 0.f;
    for (int d = lpv >> 1; d > 0; d >>= 1) ss += __shfl_xor(ss, d, 64);
    const float inv = 1.f / sqrtf(ss / (float)a.s.dv + a.eps);
    if (p >= pairs || c >= DV) return;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] *= inv * w[e] * sigmoid_acc(gate[e]);
    store8<T>(reinterpret_cast<T*>(a.out) + row * a.out_ld + h * DV + c, o);
}

// scratch of `rows` rows in segments that start anywhere: a launch holds up to rows / 16 + DELTA_MAX_SEG chunks
static size_t delta_regions(const DeltaShape& s, int rows, int es, size_t (&b)[8]) {
    const size_t n = ((size_t)rows / DELTA_C + DELTA_MAX_SEG) * s.H, C = DELTA_C;
    const size_t raw[8] = {n * C * s.DK * 4, n * C * s.DK * 4, n * C * s.DK * 4, n * s.DK * 4, n * C * C * 4, n * C * C * 4, n * C * s.DV * es, (size_t)rows * s.H * s.DV * 4};
    size_t sum = 0;
    for (int i = 0; i < 8; ++i) { b[i] = (raw[i] + 255) / 256 * 256; sum += b[i]; }
    return sum;
}
size_t delta_scratch_bytes(const DeltaShape& s, int rows, int es) { size_t b[8]; return delta_regions(s, rows, es, b); }
void delta_carve(DeltaPrefillArgs& a, void* scratch, int rows, int es) {
    size_t b[8];
    delta_regions(a.s, rows, es, b);
    char* p = static_cast<char*>(scratch);
    void* at[8];
    for (int i = 0; i < 8; ++i) { at[i] = p; p += b[i]; }
    a.kd = static_cast<float*>(at[0]); a.qd = static_cast<float*>(at[1]); a.kt = static_cast<float*>(at[2]); a.dc = static_cast<float*>(at[3]);
    a.tm = static_cast<float*>(at[4]); a.pm = static_cast<float*>(at[5]); a.v = at[6]; a.o = static_cast<float*>(at[7]);
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
    for (int i = 0, at = 0; i < a.n_seg; ++i) { LMX_REQUIRE(a.seg[i].chunk0 == at, "delta: chunks follow each other"); at += cdiv(a.seg[i].n, DELTA_C); }
    for (int i = 0; i < a.n_seg; ++i) LMX_REQUIRE(a.seg[i].n >= 1 && a.seg[i].pos0 >= 0 && a.seg[i].row0 >= 0 && a.seg[i].state && a.seg[i].ring, "delta: bad segment");
}
#define DELTA_KB(KERN, GRID, NTH, SMEM, ...) do { if (a.s.DK == 64) LMX_LAUNCH((KERN<TT, 8>), GRID, dim3(NTH), SMEM, st, __VA_ARGS__); \
                                            else if (a.s.DK == 128) LMX_LAUNCH((KERN<TT, 16>), GRID, dim3(NTH), SMEM, st, __VA_ARGS__); \
                                            else LMX_LAUNCH((KERN<TT, 32>), GRID, dim3(NTH), SMEM, st, __VA_ARGS__); } while (0)
#define DELTA_K(KERN, GRID, SMEM, ...) DELTA_KB(KERN, GRID, 256, SMEM, __VA_ARGS__)

void launch_delta_prep(int dtype, const DeltaPrefillArgs& a, hipStream_t st) {
    delta_check(a);
    int tiles = 0;
    for (int i = 0; i < a.n_seg; ++i) tiles += cdiv(a.seg[i].n, DELTA_C);
    const dim3 grid(tiles, a.s.H);
    const size_t smem = std::max((size_t)3 * DELTA_C * a.s.DK * 4, (size_t)DELTA_C * a.s.DV * dtype_size(dtype));
    LMX_REQUIRE(smem <= 60 * 1024, "delta_prep: head widths too large");
    if (dtype == kBF16) { using TT = bf16_t; DELTA_K(delta_prep_kernel, grid, smem, a); }
    else if (dtype == kF16) { using TT = f16_t; DELTA_K(delta_prep_kernel, grid, smem, a); }
    else { using TT = float; DELTA_K(delta_prep_kernel, grid, smem, a); }
    LMX_CHECK_HIP(hipGetLastError());
}
void launch_delta_scan(int dtype, const DeltaPrefillArgs& a, hipStream_t st) {
    delta_check(a);
    const dim3 grid(a.s.H * (a.s.DV / 16), a.n_seg);
    if (dtype == kBF16) { using TT = bf16_t; DELTA_K(delta_scan_kernel, grid, 0, a); }
    else if (dtype == kF16) { using TT = f16_t; DELTA_K(delta_scan_kernel, grid, 0, a); }
    else { using TT = float; DELTA_K(delta_scan_kernel, grid, 0, a); }
    LMX_CHECK_HIP(hipGetLastError());
}
void launch_delta_gate(int dtype, const DeltaPrefillArgs& a, hipStream_t st) {
    delta_check(a);
    int lpv = 8;
    while (lpv * 8 < a.s.DV) lpv <<= 1;
    LMX_REQUIRE(lpv <= 64, "delta_gate: value heads up to 512");
    for (int i = 0; i < a.n_seg;) {                          // neighbouring segments are one run of rows
        int k = i + 1, rows = a.seg[i].n;
        while (k < a.n_seg && a.seg[k].row0 == a.seg[k - 1].row0 + a.seg[k - 1].n) rows += a.seg[k++].n;
        const int pairs = rows * a.s.H;
#define L(TT) LMX_LAUNCH(delta_gate_kernel<TT>, dim3(cdiv(pairs, 256 / lpv)), dim3(256), 0, st, a, pairs, a.seg[i].row0, lpv)
        if (dtype == kBF16) L(bf16_t); else if (dtype == kF16) L(f16_t); else L(float);
#undef L
        i = k;
    }
    LMX_CHECK_HIP(hipGetLastError());
}

// ---------------------------------------------------------------------------------------------------------------
// one new token per sequence: grid (heads, sequences), 1024 threads
// ---------------------------------------------------------------------------------------------------------------
template <typename T, int LPC>
__global__ __launch_bounds__(1024) void delta_decode_kernel(DeltaDecodeArgs a) {
    constexpr int DK = LPC * 8, NTH = 1024, CPP = NTH / LPC, PF = 2;      // columns of one pass over the state, passes in flight
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ float red[NTH / 64];
    const int tid = threadIdx.x;
    const int H = a.s.H, G = a.s.G, DV = a.s.DV, taps = a.s.taps, C = a.s.channels();
    const int h = blockIdx.x, z = blockIdx.y, rep = H / G, kh = h / rep;
    float *q = sm, *k = q + DK, *g = k + DK, *v = g + DK, *gate = v + DV, *o = gate + DV;
    const DecodeFusedSeq e = a.tab ? a.tab[z] : a.one;
    const T* row = reinterpret_cast<const T*>(a.proj) + (size_t)z * a.ld;
    float* st = reinterpret_cast<float*>(e.K) + (size_t)h * DV * DK;
    T* ring = reinterpret_cast<T*>(e.VT);
    const T* conv = reinterpret_cast<const T*>(a.w.conv);
    const int sub = tid % LPC, col = tid / LPC;
    // everything that is read from memory is requested before anything waits
    float S[PF][8];
#pragma unroll
    for (int p = 0; p < PF; ++p) if (p * CPP + col < DV) load8<float>(st + (size_t)(p * CPP + col) * DK + sub * 8, S[p]);
    const int pos = *e.pos_ptr;
    const bool frozen = e.done && *e.done != 0;
    const float beta = sigmoid_acc(to_f32(row[C + h]));
    const float rate = expf(to_f32(reinterpret_cast<const T*>(a.w.A_log)[h]));
    // ---- decays and output gates: 8 lanes per row of the second low-rank matrices
    for (int i0 = tid >> 3; i0 < DK + DV; i0 += NTH / 4) {   // two rows at a time
        const T *w[2], *x[2];
        int n[2];
        float s[2] = {0.f, 0.f};
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            const int i = i0 + m * (NTH / 8);
            const bool is_g = i < DK;
            w[m] = reinterpret_cast<const T*>(a.wag) + (size_t)(is_g ? h * DK + i : H * DK + h * DV + i - DK) * a.wag_ld + (is_g ? 0 : a.ra);
            x[m] = row + a.a_off + (is_g ? 0 : a.ra);
            n[m] = i >= DK + DV ? 0 : is_g ? a.ra : a.rg;
        }
        const int most = n[0] > n[1] ? n[0] : n[1];
#pragma unroll 2
        for (int c = (tid & 7) * 8; c < most; c += 64)
#pragma unroll
            for (int m = 0; m < 2; ++m) {
                if (c >= n[m]) continue;
                float f[8], y[8]; load8<T>(w[m] + c, f); load8<T>(x[m] + c, y);
#pragma unroll
                for (int e2 = 0; e2 < 8; ++e2) s[m] = fmaf(f[e2], y[e2], s[m]);
            }
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            const int i = i0 + m * (NTH / 8);
            s[m] = round_to<T>(lanes_sum<8>(s[m]));          // the prompt path stores this product in the model dtype
            if ((tid & 7) != 0 || n[m] == 0) continue;
            if (i < DK) g[i] = decay_f32(rate, s[m] + to_f32(reinterpret_cast<const T*>(a.w.dt_bias)[h * DK + i]));
            else gate[i - DK] = sigmoid_acc(s[m]);
        }
    }
    // ---- short convolutions: thread per channel; the ring slot of this position is not one that any tap reads
    const int slot = pos % taps;
    for (int i = tid; i < 2 * DK + DV; i += NTH) {
        const bool is_v = i >= 2 * DK;
        const int c = is_v ? 2 * G * DK + h * DV + i - 2 * DK : (i < DK ? kh * DK + i : (G + kh) * DK + i - DK);
        const T xin = row[c];
        float s = to_f32(xin) * to_f32(conv[(size_t)(taps - 1) * C + c]);
        for (int j = 1, sl = slot; j < taps; ++j) {
            sl = sl == 0 ? taps - 1 : sl - 1;
            if (pos - j >= 0) s = fmaf(to_f32(ring[(size_t)sl * C + c]), to_f32(conv[(size_t)(taps - 1 - j) * C + c]), s);
        }
        if (is_v || h % rep == 0) ring[(size_t)slot * C + c] = xin;
        s = silu_acc(s);
        if (is_v) v[i - 2 * DK] = round_to<T>(s); else sm[i] = s;      // (values: the prompt path stores them in the model dtype)
    }
    __syncthreads();
    // every lane group has whole q and k: unit vectors and their product without another round
    float kr[8], qr[8], gr[8], qq = 0.f, kk = 0.f, kq = 0.f;
    load8<float>(k + sub * 8, kr); load8<float>(q + sub * 8, qr); load8<float>(g + sub * 8, gr);
#pragma unroll
    for (int n = 0; n < 8; ++n) { qq = fmaf(qr[n], qr[n], qq); kk = fmaf(kr[n], kr[n], kk); }
    qq = lanes_sum<LPC>(qq); kk = lanes_sum<LPC>(kk);
    const float qi = 1.f / (sqrtf(qq + 1e-6f) * sqrtf((float)a.s.dk)), ki = 1.f / sqrtf(kk + 1e-6f);
#pragma unroll
    for (int n = 0; n < 8; ++n) { qr[n] *= qi; kr[n] *= ki; kq = fmaf(qr[n], kr[n], kq); }
    kq = lanes_sum<LPC>(kq);
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
        const float u = beta * (v[c] - r);
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
    ss = block_sum<NTH / 64>(ss, red);                       // (its barriers also publish o)
    const float inv = 1.f / sqrtf(ss / (float)a.s.dv + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + (size_t)z * a.out_ld + h * DV;
    for (int c = tid; c < DV; c += NTH) out[c] = from_f32<T>(o[c] * inv * to_f32(reinterpret_cast<const T*>(a.w.norm)[c]) * gate[c]);
}

void launch_delta_decode(int dtype, const DeltaDecodeArgs& a, hipStream_t st) {
    delta_check(a.s);
    LMX_REQUIRE(a.ra % 64 == 0 && a.rg % 64 == 0 && a.ra >= 64 && a.rg >= 64 && a.wag_ld >= a.ra + a.rg && a.wag_ld % 8 == 0, "delta_decode: low-rank widths in whole 64-column groups");
    LMX_REQUIRE(a.a_off >= a.s.channels() + a.s.H && a.ld >= a.a_off + a.ra + a.rg, "delta_decode: bad row pitch");
    LMX_REQUIRE(a.n_seq >= 1 && (a.tab || (a.n_seq == 1 && a.one.K && a.one.VT && a.one.pos_ptr)), "delta_decode: bad sequence");
    const dim3 grid(a.s.H, a.n_seq);
    const size_t smem = (size_t)(3 * a.s.DK + 3 * a.s.DV) * 4;
    LMX_REQUIRE(smem <= 60 * 1024 && a.a_off % 8 == 0, "delta_decode: head widths too large");
    if (dtype == kBF16) { using TT = bf16_t; DELTA_KB(delta_decode_kernel, grid, 1024, smem, a); }
    else if (dtype == kF16) { using TT = f16_t; DELTA_KB(delta_decode_kernel, grid, 1024, smem, a); }
    else { using TT = float; DELTA_KB(delta_decode_kernel, grid, 1024, smem, a); }
    LMX_CHECK_HIP(hipGetLastError());
}

}  // namespace lmx
