// Kernels of the layer-list host layer (include/mi355_hybrid.h) for designs whose sublayers read the residual through a norm of their own
// and whose mixers look one token back: the step between two layers (sum of both sublayers' outputs, both norms, the mixtures of a token
// with the one before it, one launch), the low-rank decay per key channel, and the recurrence with a bonus for the current token.  The
// residual, the norms, the mixtures, the decays and the recurrence are f32.
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <math.h>

#include "common.h"
#include "hybrid_device.h"
#include "../../include/mi355_hybrid.h"

namespace {

// ------------------------------------------------------------------------------------------------------------ between two layers
struct PairStepArgs {
    const float* x; const float* y1; const float* y2; const float* rows; const int32_t* pos; const float* wts; int top;
    float* x_out; const float* n1; const float* n2; int64_t seg; float* out2_f32;
    const float* mu; int mixes; const float* h_state; int64_t state_stride; float* h_last;
    const uint32_t* ctx; const uint32_t* cu_q; const int32_t* slots; const int32_t* tok_seq;
    int width; float eps;
};
template <int E> struct Cols { float v[E]; };
template <int E> __device__ __forceinline__ Cols<E> load_cols(const float* p) {
    Cols<E> c;
    if constexpr (E == 4) { const float4 f = *reinterpret_cast<const float4*>(p); c.v[0] = f.x; c.v[1] = f.y; c.v[2] = f.z; c.v[3] = f.w; }
    else c.v[0] = *p;
    return c;
}
template <typename TO, int E> __device__ __forceinline__ void store_cols(TO* p, const Cols<E>& c) {
    if constexpr (E == 4 && sizeof(TO) == 4) *reinterpret_cast<float4*>(p) = float4{c.v[0], c.v[1], c.v[2], c.v[3]};
    else if constexpr (E == 4) *reinterpret_cast<uint2*>(p) = uint2{cvt_pk_bf16(c.v[0], c.v[1]), cvt_pk_bf16(c.v[2], c.v[3])};
    else st<TO>(p, 0, c.v[0]);
}
// A workgroup per token t: x' = x + (y1 + (y2 | the token's experts' rows)), h = x' / rms(x') n1, h2 = x' / rms(x') n2.  With mixtures the
// row before it (of the same portion) is made a second time -- x is read here and x_out written, two buffers, so no workgroup waits for
// another -- or, for a portion's first token, its h comes from the state slot (zeros at a sequence's start).
template <typename TO, int E> __global__ __launch_bounds__(1024) void pair_step_kernel(PairStepArgs p, TO* out1, TO* out2) {
    extern __shared__ __align__(16) float psm[];
    __shared__ float red[2][16];
    const int t = blockIdx.x, W = p.width, wpad = (W + 3) & ~3;
    float* xs = psm;                                     // [width] this token's new residual
    float* xp = xs + wpad;                               // [width] the one before it (mixtures only)
    float* lw = xp + (p.mixes ? wpad : 0);               // [2 top] weights of the two tokens' experts, [2 top] their rows
    int* lp = reinterpret_cast<int*>(lw + 2 * p.top);
    int s = 0, cs = 0, ce = 0, start_pos = 0;
    if (p.mixes) { s = p.tok_seq[t]; cs = (int)p.cu_q[s]; ce = (int)p.cu_q[s + 1]; start_pos = (int)p.ctx[s] - (ce - cs); }
    const bool prev = p.mixes && t > cs;
    if (p.rows) {
        for (int j = threadIdx.x; j < 2 * p.top; j += blockDim.x) {
            const int tt = j < p.top ? t : (prev ? t - 1 : t), jj = j < p.top ? j : j - p.top;
            lp[j] = p.pos[(size_t)tt * p.top + jj]; lw[j] = p.wts[(size_t)tt * p.top + jj];
        }
        __syncthreads();
    }
    auto residual = [&](int tt, int i, int o) {          // columns i .. i + E - 1 of token tt's new residual
        const size_t at = (size_t)tt * W + i;
        Cols<E> x = load_cols<E>(p.x + at), y;
#pragma unroll
        for (int e = 0; e < E; ++e) y.v[e] = 0.f;
        if (p.y1) { const Cols<E> a = load_cols<E>(p.y1 + at);
#pragma unroll
            for (int e = 0; e < E; ++e) y.v[e] += a.v[e]; }
        if (p.y2) { const Cols<E> a = load_cols<E>(p.y2 + at);
#pragma unroll
            for (int e = 0; e < E; ++e) y.v[e] += a.v[e]; }
        if (p.rows) for (int j = 0; j < p.top; ++j) {
            const Cols<E> a = load_cols<E>(p.rows + (size_t)lp[o + j] * W + i);
            const float w = lw[o + j];
#pragma unroll
            for (int e = 0; e < E; ++e) y.v[e] = fmaf(w, a.v[e], y.v[e]);
        }
#pragma unroll
        for (int e = 0; e < E; ++e) x.v[e] += y.v[e];
        return x;
    };
    float ss = 0.f, sp = 0.f;
    for (int i = threadIdx.x * E; i < W; i += blockDim.x * E) {
        const Cols<E> v = residual(t, i, 0);
        if (prev) {
            const Cols<E> b = residual(t - 1, i, p.top);
#pragma unroll
            for (int e = 0; e < E; ++e) { xp[i + e] = b.v[e]; sp = fmaf(b.v[e], b.v[e], sp); }
        }
        if (p.x_out) store_cols<float, E>(p.x_out + (size_t)t * W + i, v);
#pragma unroll
        for (int e = 0; e < E; ++e) { xs[i + e] = v.v[e]; ss = fmaf(v.v[e], v.v[e], ss); }
    }
    if (!p.n1) return;
    ss = wave_sum(ss); sp = wave_sum(sp);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    if (lane == 0) { red[0][wave] = ss; red[1][wave] = sp; }
    __syncthreads();
    ss = sp = 0.f;
    for (int w = 0; w < nw; ++w) { ss += red[0][w]; sp += red[1][w]; }
    const float inv = 1.f / sqrtf(ss / (float)W + p.eps), invp = 1.f / sqrtf(sp / (float)W + p.eps);
    const float* before = (p.mixes && !prev && start_pos > 0) ? p.h_state + (size_t)p.slots[s] * p.state_stride : nullptr;
    for (int i = threadIdx.x * E; i < W; i += blockDim.x * E) {
        const size_t at = (size_t)t * W + i;
        const Cols<E> w1 = load_cols<E>(p.n1 + i);
        Cols<E> h;
#pragma unroll
        for (int e = 0; e < E; ++e) h.v[e] = xs[i + e] * inv * w1.v[e];
        store_cols<TO, E>(out1 + at, h);
        if (p.mixes) {
            Cols<E> d;
#pragma unroll
            for (int e = 0; e < E; ++e) d.v[e] = (prev ? xp[i + e] * invp * w1.v[e] : before ? before[i + e] : 0.f) - h.v[e];
            for (int m = 0; m < p.mixes; ++m) {
                const Cols<E> mu = load_cols<E>(p.mu + (size_t)m * W + i);
                Cols<E> o;
#pragma unroll
                for (int e = 0; e < E; ++e) o.v[e] = fmaf(d.v[e], mu.v[e], h.v[e]);
                store_cols<TO, E>(out1 + (size_t)(m + 1) * p.seg + at, o);
            }
            if (t + 1 == ce) store_cols<float, E>(p.h_last + (size_t)s * W + i, h);
        }
        if (p.n2) {
            const Cols<E> w2 = load_cols<E>(p.n2 + i);
            Cols<E> g;
#pragma unroll
            for (int e = 0; e < E; ++e) g.v[e] = xs[i + e] * inv * w2.v[e];
            store_cols<TO, E>(out2 + at, g);
            if (p.out2_f32) store_cols<float, E>(p.out2_f32 + at, g);
        }
    }
}

// ------------------------------------------------------------------------------------------------------------ low-rank decay
// log w[t, c] = -exp(sum_r w2t[r, c] tanh(z[t, r]) + w0[c]).  Decoding batches: a workgroup of 256 channels and TT tokens; the tanh values
// of RC ranks at a time sit in LDS, neighbouring threads read neighbouring weights.
template <int TT> __global__ __launch_bounds__(256) void lowrank_decay_kernel(float* lw, int ldw, const float* z, int ldz, const float* w2t, const float* w0,
                                                                             int T, int R, int C) {
    constexpr int RC = 64;
    __shared__ float th[RC][TT];
    const int c = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * TT;
    float acc[TT];
    const float b = c < C ? w0[c] : 0.f;
#pragma unroll
    for (int i = 0; i < TT; ++i) acc[i] = b;
    for (int r0 = 0; r0 < R; r0 += RC) {
        const int n = min(RC, R - r0);
        __syncthreads();
        for (int i = threadIdx.x; i < RC * TT; i += 256) {
            const int tt = i / RC, r = i - tt * RC;
            th[r][tt] = (r < n && t0 + tt < T) ? tanhf(z[(size_t)(t0 + tt) * ldz + r0 + r]) : 0.f;
        }
        __syncthreads();
        if (c < C) {
            const float* w = w2t + (size_t)r0 * C + c;
            int r = 0;
            for (; r + 8 <= n; r += 8) {
                float wv[8];
#pragma unroll
                for (int u = 0; u < 8; ++u) wv[u] = w[(size_t)(r + u) * C];
#pragma unroll
                for (int u = 0; u < 8; ++u)
#pragma unroll
                    for (int i = 0; i < TT; ++i) acc[i] = fmaf(wv[u], th[r + u][i], acc[i]);
            }
            for (; r < n; ++r) {
                const float wv = w[(size_t)r * C];
#pragma unroll
                for (int i = 0; i < TT; ++i) acc[i] = fmaf(wv, th[r][i], acc[i]);
            }
        }
    }
    if (c >= C) return;
#pragma unroll
    for (int i = 0; i < TT; ++i) if (t0 + i < T) lw[(size_t)(t0 + i) * ldw + c] = -expf(acc[i]);
}

// prompts: a wave takes 16 tokens and 16 NC channels on the f32 matrix cores, its lanes make their own tanh values (operand layout of a
// 4-deep step: lane (m16, kg) holds token m16 / channel m16 at depth kg)
__device__ __forceinline__ f32x4_t mfma_f32(float a, float b, const f32x4_t& c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
template <int NC> __global__ __launch_bounds__(256) void lowrank_decay_tile_kernel(float* lw, int ldw, const float* z, int ldz, const float* w2t, const float* w0,
                                                                                  int T, int R, int C) {
    const int lane = threadIdx.x & 63, m16 = lane & 15, kg = lane >> 4;
    const int c0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * 16 * NC, t0 = blockIdx.y * 16;
    if (c0 >= C) return;
    const float* zr = z + (size_t)min(t0 + m16, T - 1) * ldz;
    int ch[NC];
    f32x4_t acc[NC];
#pragma unroll
    for (int i = 0; i < NC; ++i) {
        ch[i] = min(c0 + 16 * i + m16, C - 1);
        const float b = w0[ch[i]];
        acc[i] = f32x4_t{b, b, b, b};
    }
    constexpr int U = 4;                                 // steps whose operands are requested together
    for (int r0 = 0; r0 < R; r0 += 4 * U) {
        float a[U], w[U][NC];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int r = r0 + 4 * u + kg, rc = min(r, R - 1);
            a[u] = r < R ? zr[rc] : 0.f;
#pragma unroll
            for (int i = 0; i < NC; ++i) w[u][i] = w2t[(size_t)rc * C + ch[i]];
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const float th = tanhf(a[u]);
#pragma unroll
            for (int i = 0; i < NC; ++i) acc[i] = mfma_f32(th, w[u][i], acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < NC; ++i)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int t = t0 + 4 * kg + v;
            if (t < T && c0 + 16 * i + m16 < C) lw[(size_t)t * ldw + ch[i]] = -expf(acc[i][v]);
        }
}

// ------------------------------------------------------------------------------------------------------------ recurrence with a bonus
struct BonusArgs {
    float* o; float* state; int64_t state_stride;
    const float* rkv; int ldq, r_off, k_off, v_off; const float* lw; int ldw; const float* u;
    const uint32_t* ctx; const uint32_t* cu_q; const int32_t* slots;
    int n_seqs, H, d, vd;
    const float* row; float* row_state; int row_n;       // row != NULL: row [n_seqs, row_n] moves into the slots at row_state
};
// The thread layout of the other scans (a workgroup of 256 threads owns 256 / LPC columns of one (sequence, head)'s state [d, vd], LPC
// neighbouring lanes share a column, DP rows of it each in registers):
//   o = sum_i r_i (S_i + u_i k_i v);  S_i <- w_i S_i + k_i v
// A row's update needs the row alone; the sum over the rows is off the chain.  r, k, w of CH tokens at a time sit in LDS (the decays'
// exponentials are taken while they are staged), the next CH tokens are fetched into registers while the current ones are used.
template <int DP, int LPC, int CH> __global__ __launch_bounds__(256) void bonus_scan_kernel(BonusArgs p) {
    constexpr int RS = DP + 4, ROW = LPC * DP, TOT = CH * ROW, NPT = (TOT + 255) / 256, CPB = 256 / LPC;
    __shared__ __align__(16) float sr[2][CH][LPC][RS], sk[2][CH][LPC][RS], sw[2][CH][LPC][RS];
    const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int col = blockIdx.z * CPB + tid / LPC, part = tid % LPC;
    const int d = p.d, vd = p.vd;
    const int tb = (int)p.cu_q[s], te = (int)p.cu_q[s + 1];
    if (te <= tb) return;
    const int start_pos = (int)p.ctx[s] - (te - tb);
    const bool own = col < vd;
    float* slot = p.state + (size_t)p.slots[s] * p.state_stride;
    if (p.row && h == 0 && blockIdx.z == 0)
        for (int i = tid; i < p.row_n; i += 256) (p.row_state + (size_t)p.slots[s] * p.state_stride)[i] = p.row[(size_t)s * p.row_n + i];
    float* stt = slot + (size_t)h * d * vd;
    float S[DP], u[DP];
#pragma unroll
    for (int r = 0; r < DP; ++r) {
        const int i = part * DP + r;
        S[r] = (own && i < d && start_pos > 0) ? stt[(size_t)i * vd + col] : 0.f;
        u[r] = i < d ? p.u[h * d + i] : 0.f;
    }
    const int r_off = p.r_off + h * d, k_off = p.k_off + h * d, v_col = p.v_off + h * vd + col, w_off = h * d;
    float rr[NPT], rk[NPT], rw[NPT], rv[CH];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int n = 0; n < NPT; ++n) {
            const int idx = tid + n * 256, c = idx / ROW, ii = idx - c * ROW, t = t0 + c;
            const bool ok_ = idx < TOT && t < te && ii < d;
            const float* row = p.rkv + (size_t)(ok_ ? t : tb) * p.ldq;
            rr[n] = ok_ ? row[r_off + ii] : 0.f;
            rk[n] = ok_ ? row[k_off + ii] : 0.f;
            rw[n] = ok_ ? p.lw[(size_t)t * p.ldw + w_off + ii] : 0.f;
        }
#pragma unroll
        for (int c = 0; c < CH; ++c) rv[c] = (own && t0 + c < te) ? p.rkv[(size_t)(t0 + c) * p.ldq + v_col] : 0.f;
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int n = 0; n < NPT; ++n) {
            const int idx = tid + n * 256;
            if (idx < TOT) {
                const int c = idx / ROW, ii = idx - c * ROW, pp = ii / DP, r = ii - pp * DP;
                sr[buf][c][pp][r] = rr[n]; sk[buf][c][pp][r] = rk[n]; sw[buf][c][pp][r] = expf(rw[n]);
            }
        }
    };
    fetch(tb);
    stage(0);
    __syncthreads();
    int buf = 0;
    for (int t0 = tb; t0 < te; t0 += CH, buf ^= 1) {
        float vc[CH];
#pragma unroll
        for (int c = 0; c < CH; ++c) vc[c] = rv[c];
        const bool more = t0 + CH < te;
        if (more) fetch(t0 + CH);
        const int cn = min(CH, te - t0);
        auto token = [&](int c, float v) {
            float o = 0.f;
#pragma unroll
            for (int r = 0; r < DP; ++r) {
                const float kv = sk[buf][c][part][r] * v;
                o = fmaf(sr[buf][c][part][r], fmaf(u[r], kv, S[r]), o);
                S[r] = fmaf(sw[buf][c][part][r], S[r], kv);
            }
            o = column_sum<LPC>(o);
            if (own && part == 0) p.o[((size_t)(t0 + c) * p.H + h) * vd + col] = o;
        };
        if (cn == CH) {                                          // a whole chunk: no branch between the tokens, their LDS reads run ahead
#pragma unroll
            for (int c = 0; c < CH; ++c) token(c, vc[c]);
        } else {
#pragma unroll
            for (int c = 0; c < CH; ++c) if (c < cn) token(c, vc[c]);
        }
        if (more) stage(buf ^ 1);
        __syncthreads();
    }
    if (own)
#pragma unroll
        for (int r = 0; r < DP; ++r) { const int i = part * DP + r; if (i < d) stt[(size_t)i * vd + col] = S[r]; }
}

// ------------------------------------------------------------------------------------------------------------ the same by pieces
// Portions of prompts: the new tokens of a sequence are cut into pieces of LC tokens that are worked on side by side, a piece into
// sub-pieces of SB.  With w_t the decays per channel, E_m = the product of sub-piece m's decays, S_in the state in front of the piece:
//   prepare:  r'_t = r_t prod_(a < t) w_a,  k'_t = k_t prod_(a > t) w_a  (a in t's own sub-piece), E_m, and the scores inside a sub-piece,
//             D[t, s] = sum_i r_ti k_si prod_(s < a < t) w_ai for s < t,  D[t, t] = sum_i r_ti u_i k_ti  -- walked token by token: products of
//             decays only, no quotient of two small numbers anywhere
//   state:    U = sum_s diag(prod_(m > m(s)) E_m) k'_s v_s^T              what the piece adds to the state;  the product of all its E_m
//   scan:     S_in of the next piece = diag(prod E) S_in + U               the only sequential part, elementwise over the state
//   output:   o_t = sum_(s <= t, same sub-piece) D[t, s] v_s + sum_(s in sub-piece m < m(t)) (r'_t prod_(m < b < m(t)) E_b . k'_s) v_s
//                   + (r'_t prod_(b < m(t)) E_b) S_in
// All products run on the f32 matrix cores (16 x 16 tiles, 4 deep): the result is the recurrence's up to f32 rounding.
constexpr int LC = 64, SB = 16, NSB = LC / SB;
struct BonusPieces {
    BonusArgs a;
    float *rd, *kd, *E, *ptot, *D, *U;      // [T, H d] twice, [pieces NSB, H d], [pieces, H d], [T, H, SB], [pieces, H, d, vd]
};
// piece b of the step -> its first token and its tokens (0: past the last piece)
__device__ __forceinline__ int piece_of(const BonusArgs& p, int b, int& t0) {
    for (int s = 0; s < p.n_seqs; ++s) {
        const int tb = (int)p.cu_q[s], n = (int)p.cu_q[s + 1] - tb, pieces = (n + LC - 1) / LC;
        if (b < pieces) { t0 = tb + b * LC; return min(LC, n - b * LC); }
        b -= pieces;
    }
    return 0;
}

// a wave per sub-piece, 64 channels at a time: a lane first owns a channel (the running products of its decays), then a quarter of the
// channels of one key (the scores inside the sub-piece).  Every wave has its own part of the LDS; keys and queries pass through the same
// rows one after the other.
__device__ __forceinline__ void wave_lds_fence() {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_sched_barrier(0);
}
__global__ __launch_bounds__(256, 4) void bonus_prepare_kernel(BonusPieces q) {
    const BonusArgs& p = q.a;
    constexpr int RS = 68;                                   // floats per staged row: 64 channels + 4 of padding
    __shared__ __align__(16) float sx[NSB][SB * RS], sw[NSB][SB * RS];
    int t0;
    const int n = piece_of(p, blockIdx.x, t0), h = blockIdx.y, d = p.d, C = p.H * d;
    if (n == 0) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);       // (scalar: so are the rows' addresses)
    const int key = lane & 15, kg = lane >> 4, first = wave * SB, cnt = min(SB, n - first);
    float* X = sx[wave];
    float* Wd = sw[wave];
    float acc[SB];
#pragma unroll
    for (int t = 0; t < SB; ++t) acc[t] = 0.f;
    for (int c0 = 0; c0 < d; c0 += 64) {
        const int ch = c0 + lane;
        const bool on = ch < d;
        float r[SB], k[SB], w[SB];
        const size_t row0 = (size_t)(t0 + (cnt > 0 ? first : 0));
        const int cc = on ? ch : c0;
        const float* rp = p.rkv + row0 * p.ldq + p.r_off + h * d;
        const float* wp = p.lw + row0 * p.ldw + h * d;
        const int k_from_r = p.k_off - p.r_off;
        // (opaque copies: the addresses and comparisons below are made where they are used, not kept in registers across the chunks)
        int ld_out = C, key_ = key;
        asm volatile("" : "+s"(ld_out), "+v"(key_));
#pragma unroll
        for (int t = 0; t < SB; ++t) {                       // (rows past the portion's end: its last one again)
            r[t] = rp[cc]; k[t] = (rp + k_from_r)[cc]; w[t] = wp[cc];
            if (t + 1 < cnt) { rp += p.ldq; wp += p.ldw; }
        }
#pragma unroll
        for (int t = 0; t < SB; ++t) {
            const bool ok_ = on && t < cnt;
            r[t] = ok_ ? r[t] : 0.f; k[t] = ok_ ? k[t] : 0.f; w[t] = ok_ ? expf(w[t]) : 1.f;
        }
        wave_lds_fence();                                    // (the chunk of channels before is used up)
#pragma unroll
        for (int t = 0; t < SB; ++t) { X[t * RS + lane] = k[t]; Wd[t * RS + lane] = w[t]; }
        wave_lds_fence();
        float x[16];
        const int c4 = kg * 16;
#pragma unroll
        for (int i = 0; i < 16; i += 4) {
            const float4 kv = *reinterpret_cast<const float4*>(&X[key * RS + c4 + i]);
            x[i] = kv.x; x[i + 1] = kv.y; x[i + 2] = kv.z; x[i + 3] = kv.w;
        }
        wave_lds_fence();
        float* rd = q.rd + row0 * C + h * d;
        float* kd = q.kd + row0 * C + h * d;
        float f = 1.f;
#pragma unroll
        for (int t = 0; t < SB; ++t) {
            X[t * RS + lane] = r[t];
            if (on && t < cnt) (rd + (size_t)t * ld_out)[ch] = r[t] * f;
            f *= w[t];
        }
        if (on) q.E[((size_t)blockIdx.x * NSB + wave) * C + h * d + ch] = f;
        f = 1.f;
#pragma unroll
        for (int t = SB - 1; t >= 0; --t) {
            if (on && t < cnt) (kd + (size_t)t * ld_out)[ch] = k[t] * f;
            f *= w[t];
        }
        wave_lds_fence();
        float own = 0.f;
#pragma unroll
        for (int i = 0; i < 16; i += 4) {
            const float4 rv = *reinterpret_cast<const float4*>(&X[key * RS + c4 + i]);
            const float* u = p.u + h * d + c0 + c4 + i;
            if (c0 + c4 + i < d)
                own = fmaf(rv.x * u[0], x[i], fmaf(rv.y * u[1], x[i + 1], fmaf(rv.z * u[2], x[i + 2], fmaf(rv.w * u[3], x[i + 3], own))));
        }
#pragma unroll
        for (int t = 0; t < SB; ++t) {
            const bool past = key_ < t;
            float dot = 0.f;
#pragma unroll
            for (int i = 0; i < 16; i += 4) {
                const float4 rv = *reinterpret_cast<const float4*>(&X[t * RS + c4 + i]), wv = *reinterpret_cast<const float4*>(&Wd[t * RS + c4 + i]);
                dot = fmaf(rv.x, x[i], fmaf(rv.y, x[i + 1], fmaf(rv.z, x[i + 2], fmaf(rv.w, x[i + 3], dot))));
                x[i] *= past ? wv.x : 1.f; x[i + 1] *= past ? wv.y : 1.f; x[i + 2] *= past ? wv.z : 1.f; x[i + 3] *= past ? wv.w : 1.f;
            }
            acc[t] += past ? dot : (key_ == t ? own : 0.f);
            if (t & 1) __builtin_amdgcn_sched_barrier(0);        // (rows read further ahead than this only cost registers)
        }
    }
#pragma unroll
    for (int t = 0; t < SB; ++t) {
        float v = acc[t];
        v += __shfl_xor(v, 16);
        v += __shfl_xor(v, 32);
        if (kg == (t & 3) && t < cnt) q.D[((size_t)(t0 + first + t) * p.H + h) * SB + key] = v;
    }
}

// a wave makes 16 columns of RT 16-row tiles of U: tiles of K'^T against one of V, the whole piece's operands requested at once.  Rows past
// the portion's end read its last row against values of zero; blockIdx.z: 16 RT rows, then 64 columns.
template <int RT> __global__ __launch_bounds__(256) void bonus_state_kernel(BonusPieces q) {
    const BonusArgs& p = q.a;
    int t0;
    const int n = piece_of(p, blockIdx.x, t0), h = blockIdx.y, d = p.d, C = p.H * d;
    if (n == 0) return;
    const int row_blocks = (d + 16 * RT - 1) / (16 * RT), r0 = (blockIdx.z % row_blocks) * 16 * RT;
    const float* E = q.E + (size_t)blockIdx.x * NSB * C + h * d;
    if (blockIdx.z == 0)
        for (int i = threadIdx.x; i < d; i += blockDim.x) {
            float f = 1.f;
#pragma unroll
            for (int b = 0; b < NSB; ++b) if (b * SB < n) f *= E[(size_t)b * C + i];
            q.ptot[(size_t)blockIdx.x * C + h * d + i] = f;
        }
    const int lane = threadIdx.x & 63, m16 = lane & 15, kg = lane >> 4, col = ((blockIdx.z / row_blocks) * 4 + (threadIdx.x >> 6)) * 16 + m16;
    if (col - m16 >= p.vd) return;
    const float* K = q.kd + (size_t)t0 * C + h * d + m16;
    const float* V = p.rkv + (size_t)t0 * p.ldq + p.v_off + h * p.vd + col;
    float* U = q.U + ((size_t)blockIdx.x * p.H + h) * d * p.vd;
    float a[NSB][4][RT], v[NSB][4], e[NSB][RT];
#pragma unroll
    for (int b = 0; b < NSB; ++b) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int t = b * SB + 4 * j + kg, tc = min(t, n - 1);
            v[b][j] = V[(size_t)tc * p.ldq];
            v[b][j] = t < n ? v[b][j] : 0.f;
#pragma unroll
            for (int i = 0; i < RT; ++i) a[b][j][i] = K[(size_t)tc * C + min(r0 + 16 * i, d - 16)];
        }
#pragma unroll
        for (int i = 0; i < RT; ++i) e[b][i] = b * SB < n ? E[(size_t)b * C + min(r0 + 16 * i, d - 16) + m16] : 1.f;
    }
    f32x4_t acc[RT];
    float f[RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) { acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f}; f[i] = 1.f; }
#pragma unroll
    for (int b = NSB - 1; b >= 0; --b) {                     // from the piece's end: the factor of a sub-piece is the product of those behind it
        if (b * SB < n)
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int i = 0; i < RT; ++i) acc[i] = mfma_f32(a[b][j][i] * f[i], v[b][j], acc[i]);
#pragma unroll
        for (int i = 0; i < RT; ++i) f[i] *= e[b][i];
    }
#pragma unroll
    for (int i = 0; i < RT; ++i)
        if (r0 + 16 * i < d)
#pragma unroll
            for (int x = 0; x < 4; ++x) U[(size_t)(r0 + 16 * i + 4 * kg + x) * p.vd + col] = acc[i][x];
}

// a thread per element of a (sequence, head)'s state: the states in front of its pieces, then the one behind the last
__global__ __launch_bounds__(256) void bonus_piece_scan_kernel(BonusPieces q) {
    const BonusArgs& p = q.a;
    const int s = blockIdx.x, h = blockIdx.y, e = blockIdx.z * 256 + threadIdx.x, per = p.d * p.vd;
    const int n = (int)p.cu_q[s + 1] - (int)p.cu_q[s];
    if (n <= 0) return;
    if (p.row && h == 0)
        for (int i = e; i < p.row_n; i += gridDim.z * 256) (p.row_state + (size_t)p.slots[s] * p.state_stride)[i] = p.row[(size_t)s * p.row_n + i];
    if (e >= per) return;
    int first = 0;
    for (int i = 0; i < s; ++i) first += ((int)p.cu_q[i + 1] - (int)p.cu_q[i] + LC - 1) / LC;
    const int pieces = (n + LC - 1) / LC;
    float* stt = p.state + (size_t)p.slots[s] * p.state_stride + (size_t)h * per + e;
    float S = (int)p.ctx[s] > n ? *stt : 0.f;
    const size_t step = (size_t)p.H * per, fstep = (size_t)p.H * p.d;
    float* u = q.U + (size_t)first * step + (size_t)h * per + e;
    const float* f = q.ptot + (size_t)first * fstep + h * p.d + e / p.vd;
    constexpr int AHEAD = 8;                      // pieces whose contributions are requested together
    for (int c0 = 0; c0 < pieces; c0 += AHEAD) {
        float add[AHEAD], mul[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) { add[i] = c0 + i < pieces ? u[(size_t)(c0 + i) * step] : 0.f; mul[i] = c0 + i < pieces ? f[(size_t)(c0 + i) * fstep] : 0.f; }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i)
            if (c0 + i < pieces) { u[(size_t)(c0 + i) * step] = S; S = fmaf(mul[i], S, add[i]); }
    }
    *stt = S;
}

// a wave takes the 16 queries of one sub-piece and 16 VT columns of the output: its scores against the sub-pieces before it and the ones
// inside it through LDS into the layout of a left operand, then the two products into one accumulator.  (The depth of a product is walked
// in the order 16 j + 4 kg + e, e innermost, on both operands: rows are read 16 bytes at a time.)
template <int VT> __global__ __launch_bounds__(256, VT <= 4 ? 3 : 2) void bonus_output_kernel(BonusPieces q) {
    const BonusArgs& p = q.a;
    constexpr int PR = LC + 4;
    __shared__ __align__(16) float P[NSB][SB * PR];
    int t0;
    const int n = piece_of(p, blockIdx.x, t0), h = blockIdx.y;
    if (n == 0) return;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m16 = lane & 15, kg = lane >> 4, row0 = SB * wave;
    if (row0 >= n) return;
    const int d = p.d, vd = p.vd, C = p.H * d, col0 = blockIdx.z * 16 * VT;
    const float* R = q.rd + (size_t)(t0 + min(row0 + m16, n - 1)) * C + h * d + 4 * kg;
    const float* K = q.kd + (size_t)(t0 + m16) * C + h * d + 4 * kg;
    const float* E = q.E + (size_t)blockIdx.x * NSB * C + h * d + 4 * kg;
    const float* V = p.rkv + (size_t)t0 * p.ldq + p.v_off + h * vd + col0 + m16;
    const float* S = q.U + ((size_t)blockIdx.x * p.H + h) * d * vd + col0 + m16;
    f32x4_t sc[NSB - 1], acc[VT];
#pragma unroll
    for (int i = 0; i < NSB - 1; ++i) sc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < VT; ++c) acc[c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    // (the operands of the next 16 of the depth are requested before the current ones are multiplied)
    float4 rn, kn[NSB - 1], en[NSB - 1], k[NSB - 1], e4[NSB - 1];
    float b[4][VT], bn[4][VT];
    auto fetch = [&](int j) {
        rn = *reinterpret_cast<const float4*>(R + j);
#pragma unroll
        for (int i = 0; i < NSB - 1; ++i)
            if (i < wave) { kn[i] = *reinterpret_cast<const float4*>(K + (size_t)i * SB * C + j); en[i] = *reinterpret_cast<const float4*>(E + (size_t)i * C + j); }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int c = 0; c < VT; ++c) bn[e][c] = col0 + 16 * c < vd ? S[(size_t)(j + 4 * kg + e) * vd + 16 * c] : 0.f;
    };
    auto fetch_values = [&](int j) {
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int c = 0; c < VT; ++c) {
                const int t = j + 4 * kg + e;
                bn[e][c] = (t < n && col0 + 16 * c < vd) ? V[(size_t)t * p.ldq + 16 * c] : 0.f;
            }
    };
    auto take = [&]() {
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int c = 0; c < VT; ++c) b[e][c] = bn[e][c];
    };
    fetch(0);
    float* Pw = P[wave];
    for (int v = 0; v < 4; ++v) {                            // the scores inside the sub-piece (rows past the portion's end are not stored below)
        const int r = min(row0 + 4 * kg + v, n - 1);
        Pw[(4 * kg + v) * PR + row0 + m16] = q.D[((size_t)(t0 + r) * p.H + h) * SB + m16];
    }
    for (int j = 0; j < d; j += 16) {
        float g[4] = {rn.x, rn.y, rn.z, rn.w};
#pragma unroll
        for (int i = 0; i < NSB - 1; ++i) { k[i] = kn[i]; e4[i] = en[i]; }
        take();
        if (j + 16 < d) fetch(j + 16); else fetch_values(0);
#pragma unroll
        for (int i = NSB - 2; i >= 0; --i) {                 // from the sub-piece before this one back to the piece's first
            if (i >= wave) continue;
            const float ka[4] = {k[i].x, k[i].y, k[i].z, k[i].w}, ea[4] = {e4[i].x, e4[i].y, e4[i].z, e4[i].w};
#pragma unroll
            for (int e = 0; e < 4; ++e) sc[i] = mfma_f32(g[e], ka[e], sc[i]);
#pragma unroll
            for (int e = 0; e < 4; ++e) g[e] *= ea[e];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int c = 0; c < VT; ++c) acc[c] = mfma_f32(g[e], b[e][c], acc[c]);
    }
#pragma unroll
    for (int i = 0; i < NSB - 1; ++i)
        if (i < wave)
#pragma unroll
            for (int v = 0; v < 4; ++v) Pw[(4 * kg + v) * PR + SB * i + m16] = sc[i][v];
    wave_lds_fence();
    for (int j = 0; j <= row0; j += 16) {
        take();
        if (j + 16 <= row0) fetch_values(j + 16);
        const float4 a4 = *reinterpret_cast<const float4*>(&Pw[m16 * PR + j + 4 * kg]);
        const float a[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int c = 0; c < VT; ++c) acc[c] = mfma_f32(a[e], b[e][c], acc[c]);
    }
#pragma unroll
    for (int c = 0; c < VT; ++c) {
        if (col0 + 16 * c >= vd) break;
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int r = row0 + 4 * kg + v;
            if (r < n) p.o[((size_t)(t0 + r) * p.H + h) * vd + col0 + 16 * c + m16] = acc[c][v];
        }
    }
}

template <typename TO> int pair_launch(const PairStepArgs& p, TO* out1, TO* out2, int T, hipStream_t s_) {
    auto aligned = [](const void* q) { return (uintptr_t)q % 16 == 0; };
    const bool vec = p.width % 4 == 0 && p.seg % 4 == 0 && aligned(p.x) && aligned(p.y1) && aligned(p.y2) && aligned(p.rows) &&
                     aligned(p.x_out) && aligned(out1) && aligned(out2) && aligned(p.out2_f32) && aligned(p.n1) && aligned(p.n2) && aligned(p.mu) &&
                     aligned(p.h_last);
    const int items = vec ? p.width / 4 : p.width;
    // few rows (decoding batches): a thread per item so that a row's loads are in flight together; prompts: four waves a row
    const int nt = T <= 64 ? min(1024, max(64, (items + 63) / 64 * 64)) : 256;
    const size_t lds = ((size_t)((p.width + 3) & ~3) * (p.mixes ? 2 : 1) + 4 * (size_t)p.top) * 4;
    if (lds > 65536) {
        const hipError_t e = vec ? hipFuncSetAttribute(reinterpret_cast<const void*>(&pair_step_kernel<TO, 4>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)
                                 : hipFuncSetAttribute(reinterpret_cast<const void*>(&pair_step_kernel<TO, 1>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
    }
    if (vec) pair_step_kernel<TO, 4><<<T, nt, lds, s_>>>(p, out1, out2);
    else pair_step_kernel<TO, 1><<<T, nt, lds, s_>>>(p, out1, out2);
    return 0;
}

}  // namespace

extern "C" {

int mi355_hyb_pair_step(const float* x, const float* y1, const float* y2, const float* moe_rows, const int32_t* moe_pos, const float* moe_w,
                        int32_t top, float* x_out, const float* norm1, const float* norm2, void* out1, int64_t seg_stride, void* out2,
                        int32_t out_dtype, float* out2_f32, const float* mu, int32_t mixes, const float* h_state, int64_t state_stride,
                        float* h_last, const uint32_t* context_lens, const uint32_t* cu_seqlens_q, const int32_t* state_slots,
                        const int32_t* token_seq, int32_t T, int32_t width, float eps, int64_t stream) {
    if (!x || width <= 0 || width > 16384 || mixes < 0 || (!x_out && !norm1)) return -1;
    if (norm1 && (!out1 || !is_dt(out_dtype) || (norm2 && !out2))) return -1;
    if (moe_rows && (!moe_pos || !moe_w || top < 1 || top > 1024)) return -1;
    if (!norm1) mixes = 0;
    if (mixes && (!mu || !h_state || !h_last || !context_lens || !cu_seqlens_q || !state_slots || !token_seq || x_out == x || seg_stride < (int64_t)T * width)) return -1;
    if (T <= 0) return 0;
    PairStepArgs p{x, y1, y2, moe_rows, moe_pos, moe_w, moe_rows ? top : 0, x_out, norm1, norm2, seg_stride, out2_f32, mu, mixes, h_state, state_stride,
                   h_last, context_lens, cu_seqlens_q, state_slots, token_seq, width, eps};
    const int rc = (!norm1 || out_dtype == MI355_DTYPE_F32) ? pair_launch<float>(p, (float*)out1, (float*)out2, T, to_stream(stream))
                                                            : pair_launch<uint16_t>(p, (uint16_t*)out1, (uint16_t*)out2, T, to_stream(stream));
    if (rc != 0) return rc;
    LAUNCH_OK(); return 0;
}

int mi355_hyb_lowrank_decay(float* log_w, int32_t ldw, const float* z, int32_t ldz, const float* w2t, const float* w0, int32_t T, int32_t rank,
                            int32_t channels, int64_t stream) {
    if (!log_w || !z || !w2t || !w0 || rank <= 0 || channels <= 0 || ldw < channels || ldz < rank) return -1;
    if (T <= 0) return 0;
    hipStream_t s_ = to_stream(stream);
    if (T <= 64) lowrank_decay_kernel<1><<<dim3((unsigned)((channels + 255) / 256), T), 256, 0, s_>>>(log_w, ldw, z, ldz, w2t, w0, T, rank, channels);
    else lowrank_decay_tile_kernel<8><<<dim3((unsigned)((channels + 511) / 512), (T + 15) / 16), 256, 0, s_>>>(log_w, ldw, z, ldz, w2t, w0, T, rank, channels);
    LAUNCH_OK(); return 0;
}

int64_t mi355_hyb_bonus_recurrence_scratch(int32_t num_tokens, int32_t num_seqs, int32_t heads, int32_t dim, int32_t vdim) {
    if (num_tokens < LC || num_tokens <= 8 * (int64_t)num_seqs || heads <= 0 || dim <= 0 || vdim <= 0 || dim % 16 || vdim % 16 || dim > 512) return 0;
    const int64_t C = (int64_t)heads * dim, np = (int64_t)num_tokens / LC + num_seqs;
    return 2 * num_tokens * C + np * (NSB + 1) * C + (int64_t)num_tokens * heads * SB + np * C * vdim;
}

int mi355_hyb_bonus_recurrence(float* o, float* state, int64_t state_stride, const float* rkv, int32_t ldq, int32_t r_off, int32_t k_off,
                               int32_t v_off, const float* log_w, int32_t ldw, const float* bonus, const uint32_t* context_lens,
                               const uint32_t* cu_seqlens_q, const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t heads,
                               int32_t dim, int32_t vdim, const float* row, float* row_state, int32_t row_n, float* scratch, int64_t stream) {
    if (!o || !state || !rkv || !log_w || !bonus || !context_lens || !cu_seqlens_q || !state_slots || (row && (!row_state || row_n <= 0))) return -1;
    if (heads <= 0 || heads > 65535 || dim <= 0 || dim > 512 || vdim <= 0 || r_off < 0 || k_off < 0 || v_off < 0 || ldw < heads * dim) return -1;
    if (ldq < r_off + heads * dim || ldq < k_off + heads * dim || ldq < v_off + heads * vdim) return -1;
    if (num_seqs <= 0 || num_tokens <= 0) return 0;
    BonusArgs p{o, state, state_stride, rkv, ldq, r_off, k_off, v_off, log_w, ldw, bonus, context_lens, cu_seqlens_q, state_slots, num_seqs, heads, dim,
                vdim, row, row_state, row_n};
    hipStream_t s_ = to_stream(stream);
    if (scratch && dim % 16 == 0 && vdim % 16 == 0 && (uintptr_t)scratch % 16 == 0) {
        const size_t C = (size_t)heads * dim, np = (size_t)num_tokens / LC + num_seqs;
        BonusPieces q{p, scratch, scratch + num_tokens * C};
        q.E = q.kd + num_tokens * C;
        q.ptot = q.E + np * NSB * C;
        q.D = q.ptot + np * C;
        q.U = q.D + (size_t)num_tokens * heads * SB;
        const dim3 pg((unsigned)np, heads);
        bonus_prepare_kernel<<<pg, 256, 0, s_>>>(q);
        bonus_state_kernel<4><<<dim3((unsigned)np, heads, ((dim + 63) / 64) * ((vdim + 63) / 64)), 256, 0, s_>>>(q);
        bonus_piece_scan_kernel<<<dim3(num_seqs, heads, (dim * vdim + 255) / 256), 256, 0, s_>>>(q);
        if (vdim <= 32) bonus_output_kernel<2><<<pg, 256, 0, s_>>>(q);
        else if (vdim <= 64) bonus_output_kernel<4><<<pg, 256, 0, s_>>>(q);
        else bonus_output_kernel<8><<<dim3((unsigned)np, heads, (vdim + 127) / 128), 256, 0, s_>>>(q);
        LAUNCH_OK(); return 0;
    }
    if (dim < 64) {
        const dim3 grid(num_seqs, heads, (vdim + 63) / 64);
        if (dim <= 16) bonus_scan_kernel<4, 4, 8><<<grid, 256, 0, s_>>>(p);
        else if (dim <= 32) bonus_scan_kernel<8, 4, 8><<<grid, 256, 0, s_>>>(p);
        else bonus_scan_kernel<16, 4, 8><<<grid, 256, 0, s_>>>(p);
    } else {
        const dim3 grid(num_seqs, heads, (vdim + 15) / 16);
        if (dim <= 64) { if (num_tokens > 8 * num_seqs) bonus_scan_kernel<4, 16, 16><<<grid, 256, 0, s_>>>(p); else bonus_scan_kernel<4, 16, 8><<<grid, 256, 0, s_>>>(p); }
        else if (dim <= 128) bonus_scan_kernel<8, 16, 8><<<grid, 256, 0, s_>>>(p);
        else if (dim <= 256) bonus_scan_kernel<16, 16, 8><<<grid, 256, 0, s_>>>(p);
        else bonus_scan_kernel<32, 16, 2><<<grid, 256, 0, s_>>>(p);
    }
    LAUNCH_OK(); return 0;
}

}  // extern "C"
