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
// log w[t, c] = -exp(sum_r w2t[r, c] tanh(z[t, r]) + w0[c]).  A workgroup of 256 channels and TT tokens; the tanh values of RC ranks at a
// time sit in LDS, neighbouring threads read neighbouring weights.
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
    const unsigned nx = (unsigned)((channels + 255) / 256);
    if (T <= 64) lowrank_decay_kernel<1><<<dim3(nx, T), 256, 0, s_>>>(log_w, ldw, z, ldz, w2t, w0, T, rank, channels);
    else lowrank_decay_kernel<16><<<dim3(nx, (T + 15) / 16), 256, 0, s_>>>(log_w, ldw, z, ldz, w2t, w0, T, rank, channels);
    LAUNCH_OK(); return 0;
}

int mi355_hyb_bonus_recurrence(float* o, float* state, int64_t state_stride, const float* rkv, int32_t ldq, int32_t r_off, int32_t k_off,
                               int32_t v_off, const float* log_w, int32_t ldw, const float* bonus, const uint32_t* context_lens,
                               const uint32_t* cu_seqlens_q, const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t heads,
                               int32_t dim, int32_t vdim, const float* row, float* row_state, int32_t row_n, float* scratch, int64_t stream) {
    if (!o || !state || !rkv || !log_w || !bonus || !context_lens || !cu_seqlens_q || !state_slots || (row && (!row_state || row_n <= 0))) return -1;
    if (heads <= 0 || heads > 65535 || dim <= 0 || dim > 512 || vdim <= 0 || r_off < 0 || k_off < 0 || v_off < 0 || ldw < heads * dim) return -1;
    if (ldq < r_off + heads * dim || ldq < k_off + heads * dim || ldq < v_off + heads * vdim) return -1;
    if (num_seqs <= 0 || num_tokens <= 0) return 0;
    (void)scratch;
    BonusArgs p{o, state, state_stride, rkv, ldq, r_off, k_off, v_off, log_w, ldw, bonus, context_lens, cu_seqlens_q, state_slots, num_seqs, heads, dim,
                vdim, row, row_state, row_n};
    hipStream_t s_ = to_stream(stream);
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
