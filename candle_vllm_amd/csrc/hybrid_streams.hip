// Kernels of the layer-list host layer (include/mi355_hybrid.h) for designs whose residual stream is carried in several copies: the step
// between two sublayers (experts' sum, mixing of the copies, the next sublayer's input and its norm, one launch), the embedding with a
// row per pair of neighbouring tokens, and the norm with a sigmoid gate behind it.  The copies, the mixing and the norms are f32.
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <math.h>

#include "common.h"
#include "hybrid_device.h"
#include "../../include/mi355_hybrid.h"

namespace {

// One workgroup per sequence: the word of the state slot is read for the portion's first token before it is replaced by the last one.
__global__ __launch_bounds__(256) void bigram_rows_kernel(int32_t* rows, int32_t* last, int64_t stride, const uint32_t* tokens, const uint32_t* ctx,
                                                          const uint32_t* cu_q, const int32_t* slots, int buckets, int64_t mul_prev, int64_t mul_cur) {
    const int s = blockIdx.x, tb = (int)cu_q[s], te = (int)cu_q[s + 1];
    if (te <= tb) return;
    int32_t* word = last + (size_t)slots[s] * stride;
    const bool fresh = (int)ctx[s] == te - tb;
    const uint32_t before = fresh ? 0u : (uint32_t)*word;
    __syncthreads();
    for (int t = tb + threadIdx.x; t < te; t += blockDim.x) {
        const uint64_t prev = t > tb ? tokens[t - 1] : before;
        const uint64_t h = prev * (uint64_t)mul_prev + (uint64_t)tokens[t] * (uint64_t)mul_cur;
        rows[t] = (t == tb && fresh) ? buckets : (int)(h % (uint64_t)buckets);
    }
    if (threadIdx.x == 0) *word = (int32_t)tokens[te - 1];
}

template <typename TW> __global__ __launch_bounds__(1024) void embed_streams_kernel(float* x, const TW* table, const TW* bigram, const int32_t* rows, const uint32_t* ids,
                                                            int copies, int width, int vocab, float scale) {
    const int t = blockIdx.x;
    const uint32_t id = min(ids[t], (uint32_t)(vocab - 1));
    const TW* br = bigram ? bigram + (size_t)rows[t] * width : nullptr;
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        float v = ld<TW>(table, (size_t)id * width + i) * scale;
        if (br) v += ld<TW>(br, i);
        for (int s = 0; s < copies; ++s) x[((size_t)t * copies + s) * width + i] = v;
    }
}

struct StreamArgs {
    float* X; const float* y; const float* rows; const int32_t* pos; const float* wts; int top;
    const float* mix; const float* ow; float* sum; const float* iw; const float* nw; float* out_f32;
    int S, width; float eps;
};
// A workgroup per token: every thread carries E neighbouring columns of all copies through the mixing (a column of the copies depends on
// the same column only), keeps the next sublayer's input in LDS and comes back to it once the row's mean square is known.  The weights
// of the mixing are the same for the whole grid; up to 4 copies they sit in registers, beyond that in LDS.
template <typename TO, int SM, int E> __global__ __launch_bounds__(1024) void stream_step_kernel(StreamArgs p, TO* out) {
    extern __shared__ __align__(16) float ssm[];
    __shared__ float red[16];
    float* us = ssm;                                        // [width]: the next sublayer's input
    float* lm = us + ((p.width + 3) & ~3);                  // [SM SM] mixing, [SM] output, [SM] input weights
    float* lw = lm + SM * SM + 2 * SM;                      // [top] weights, [top] rows of the token's experts
    int* lp = reinterpret_cast<int*>(lw + p.top);
    const int t = blockIdx.x, S = p.S, W = p.width;
    for (int i = threadIdx.x; i < SM * SM + 2 * SM; i += blockDim.x) {
        float v = 0.f;
        if (i < SM * SM) { const int a = i / SM, b = i % SM; if (p.mix && a < S && b < S) v = p.mix[a * S + b]; }
        else if (i < SM * SM + SM) { if (p.mix && i - SM * SM < S) v = p.ow[i - SM * SM]; }
        else if (p.nw && i - SM * SM - SM < S) v = p.iw[i - SM * SM - SM];
        lm[i] = v;
    }
    if (p.rows) for (int j = threadIdx.x; j < p.top; j += blockDim.x) { lp[j] = p.pos[(size_t)t * p.top + j]; lw[j] = p.wts[(size_t)t * p.top + j]; }
    __syncthreads();
    constexpr bool REG = SM <= 4;
    float rm[REG ? SM * SM + 2 * SM : 1];
    if (REG)
#pragma unroll
        for (int i = 0; i < SM * SM + 2 * SM; ++i) rm[REG ? i : 0] = lm[i];
    auto wt = [&](int i) { return REG ? rm[REG ? i : 0] : lm[i]; };
    float* X = p.X + (size_t)t * S * W;
    float ss = 0.f;
    for (int i = threadIdx.x * E; i < W; i += blockDim.x * E) {
        float x[SM][E];
#pragma unroll
        for (int s = 0; s < SM; ++s) {
            if (s < S) {
                if (E == 4) { const float4 v = *reinterpret_cast<const float4*>(X + (size_t)s * W + i); x[s][0] = v.x; x[s][1 % E] = v.y; x[s][2 % E] = v.z; x[s][3 % E] = v.w; }
                else x[s][0] = X[(size_t)s * W + i];
            } else {
#pragma unroll
                for (int e = 0; e < E; ++e) x[s][e] = 0.f;
            }
        }
        if (p.mix) {
            float y[E];
#pragma unroll
            for (int e = 0; e < E; ++e) y[e] = 0.f;
            auto take = [&](const float* row, float w) {
                if (E == 4) { const float4 v = *reinterpret_cast<const float4*>(row); y[0] = fmaf(w, v.x, y[0]); y[1 % E] = fmaf(w, v.y, y[1 % E]); y[2 % E] = fmaf(w, v.z, y[2 % E]); y[3 % E] = fmaf(w, v.w, y[3 % E]); }
                else y[0] = fmaf(w, *row, y[0]);
            };
            if (p.y) take(p.y + (size_t)t * W + i, 1.f);
            if (p.rows) for (int j = 0; j < p.top; ++j) take(p.rows + (size_t)lp[j] * W + i, lw[j]);
            float nx[SM][E];
#pragma unroll
            for (int b = 0; b < SM; ++b)
#pragma unroll
                for (int e = 0; e < E; ++e) {
                    float a = wt(SM * SM + b) * y[e];
#pragma unroll
                    for (int s = 0; s < SM; ++s) a = fmaf(wt(s * SM + b), x[s][e], a);
                    nx[b][e] = a;
                }
#pragma unroll
            for (int s = 0; s < SM; ++s)
#pragma unroll
                for (int e = 0; e < E; ++e) x[s][e] = nx[s][e];
            if (p.nw)
#pragma unroll
                for (int s = 0; s < SM; ++s) {
                    if (s >= S) break;
                    if (E == 4) *reinterpret_cast<float4*>(X + (size_t)s * W + i) = float4{x[s][0], x[s][1 % E], x[s][2 % E], x[s][3 % E]};
                    else X[(size_t)s * W + i] = x[s][0];
                }
        }
        if (p.sum)
#pragma unroll
            for (int e = 0; e < E; ++e) {
                float a = 0.f;
#pragma unroll
                for (int s = 0; s < SM; ++s) a += x[s][e];          // (copies beyond S are zero)
                p.sum[(size_t)t * W + i + e] = a;
            }
        if (p.nw)
#pragma unroll
            for (int e = 0; e < E; ++e) {
                float u = 0.f;
#pragma unroll
                for (int s = 0; s < SM; ++s) u = fmaf(wt(SM * SM + SM + s), x[s][e], u);
                us[i + e] = u;
                ss = fmaf(u, u, ss);
            }
    }
    if (!p.nw) return;
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)W + p.eps);
    for (int i = threadIdx.x * E; i < W; i += blockDim.x * E) {
#pragma unroll
        for (int e = 0; e < E; ++e) {
            const float v = us[i + e] * inv * p.nw[i + e];
            st<TO>(out, (size_t)t * W + i + e, v);
            if (p.out_f32) p.out_f32[(size_t)t * W + i + e] = v;
        }
    }
}

// out = y / rms(y over the part) * w * sigmoid(z): a workgroup per (token, part)
template <typename TO> __global__ __launch_bounds__(1024) void norm_sigmoid_gate_kernel(TO* out, const float* y, const float* gate_in, int ldg, const float* w,
                                                                                       int n, int groups, float eps) {
    __shared__ float red[16];
    const int t = blockIdx.x, per = n / groups, c0 = blockIdx.y * per;
    const float* yr = y + (size_t)t * n + c0;
    const float* zr = gate_in + (size_t)t * ldg + c0;
    float ss = 0.f;
    for (int i = threadIdx.x; i < per; i += blockDim.x) ss = fmaf(yr[i], yr[i], ss);
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)per + eps);
    for (int i = threadIdx.x; i < per; i += blockDim.x) st<TO>(out, (size_t)t * n + c0 + i, yr[i] * inv * w[c0 + i] * sigmoidf_(zr[i]));
}

template <typename TO, int SM> void stream_launch(const StreamArgs& p, TO* out, int T, hipStream_t s_) {
    const bool vec = p.width % 4 == 0 && (uintptr_t)p.X % 16 == 0 && (uintptr_t)p.y % 16 == 0 && (uintptr_t)p.rows % 16 == 0;
    const int items = vec ? p.width / 4 : p.width;
    // few rows (decoding batches): a thread per item so that a row's loads are in flight together; prompts: four waves a row
    const int nt = T <= 64 ? min(1024, max(64, (items + 63) / 64 * 64)) : 256;
    const size_t lds = ((size_t)((p.width + 3) & ~3) + SM * SM + 2 * SM + 2 * (size_t)p.top) * 4;
    if (vec) stream_step_kernel<TO, SM, 4><<<T, nt, lds, s_>>>(p, out);
    else stream_step_kernel<TO, SM, 1><<<T, nt, lds, s_>>>(p, out);
}
template <typename TO> void stream_dispatch(const StreamArgs& p, TO* out, int T, hipStream_t s_) {
    if (p.S == 1) stream_launch<TO, 1>(p, out, T, s_);
    else if (p.S == 2) stream_launch<TO, 2>(p, out, T, s_);
    else if (p.S <= 4) stream_launch<TO, 4>(p, out, T, s_);
    else if (p.S <= 8) stream_launch<TO, 8>(p, out, T, s_);
    else stream_launch<TO, 16>(p, out, T, s_);
}

}  // namespace

extern "C" {

int mi355_hyb_bigram_rows(int32_t* rows, int32_t* last_token, int64_t state_stride, const uint32_t* tokens, const uint32_t* context_lens,
                          const uint32_t* cu_seqlens_q, const int32_t* state_slots, int32_t num_seqs, int32_t num_tokens, int32_t buckets,
                          int64_t mul_prev, int64_t mul_cur, int64_t stream) {
    if (!rows || !last_token || !tokens || !context_lens || !cu_seqlens_q || !state_slots || buckets < 1 || mul_prev < 0 || mul_cur < 0) return -1;
    if (num_seqs <= 0 || num_tokens <= 0) return 0;
    bigram_rows_kernel<<<num_seqs, 256, 0, to_stream(stream)>>>(rows, last_token, state_stride, tokens, context_lens, cu_seqlens_q, state_slots, buckets,
                                                               mul_prev, mul_cur);
    LAUNCH_OK(); return 0;
}

int mi355_hyb_embed_streams(float* x, const void* table, const void* bigram, const int32_t* bigram_rows, const uint32_t* ids, int32_t T,
                            int32_t copies, int32_t width, int32_t vocab, float scale, int32_t dtype, int64_t stream) {
    if (!x || !table || !ids || (bigram && !bigram_rows) || copies < 1 || width <= 0 || vocab <= 0 || !is_dt(dtype)) return -1;
    if (T <= 0) return 0;
    hipStream_t s_ = to_stream(stream);
    const int nt = (T <= 64 && width > 256) ? 1024 : 256;
    if (dtype == MI355_DTYPE_F32) embed_streams_kernel<float><<<T, nt, 0, s_>>>(x, (const float*)table, (const float*)bigram, bigram_rows, ids, copies, width, vocab, scale);
    else embed_streams_kernel<uint16_t><<<T, nt, 0, s_>>>(x, (const uint16_t*)table, (const uint16_t*)bigram, bigram_rows, ids, copies, width, vocab, scale);
    LAUNCH_OK(); return 0;
}

int mi355_hyb_stream_step(float* X, const float* y_dense, const float* moe_rows, const int32_t* moe_pos, const float* moe_w, int32_t top,
                          const float* mix, const float* out_w, float* sum, const float* in_w, const float* norm_w, void* out,
                          int32_t out_dtype, float* out_f32, int32_t T, int32_t streams, int32_t width, float eps, int64_t stream) {
    if (!X || streams < 1 || streams > 16 || width <= 0 || width > 12288 || (mix && !out_w)) return -1;
    if (moe_rows && (!moe_pos || !moe_w || top < 1 || top > 1024)) return -1;
    if (norm_w && (!in_w || !out || !is_dt(out_dtype))) return -1;
    if (T <= 0) return 0;
    StreamArgs p{X, y_dense, moe_rows, moe_pos, moe_w, moe_rows ? top : 0, mix, out_w, sum, in_w, norm_w, out_f32, streams, width, eps};
    if (!norm_w || out_dtype == MI355_DTYPE_F32) stream_dispatch<float>(p, (float*)out, T, to_stream(stream));
    else stream_dispatch<uint16_t>(p, (uint16_t*)out, T, to_stream(stream));
    LAUNCH_OK(); return 0;
}

int mi355_hyb_norm_sigmoid_gate(void* out, int32_t out_dtype, const float* y, const float* gate_in, int32_t ldg, const float* w, int32_t T,
                                int32_t n, int32_t groups, float eps, int64_t stream) {
    if (!out || !y || !gate_in || !w || !is_dt(out_dtype) || n <= 0 || groups < 1 || n % groups || ldg < n) return -1;
    if (T <= 0) return 0;
    const dim3 grid(T, groups);
    const int nt = (T <= 64 && n / groups > 256) ? 1024 : 256;
    if (out_dtype == MI355_DTYPE_F32) norm_sigmoid_gate_kernel<float><<<grid, nt, 0, to_stream(stream)>>>((float*)out, y, gate_in, ldg, w, n, groups, eps);
    else norm_sigmoid_gate_kernel<uint16_t><<<grid, nt, 0, to_stream(stream)>>>((uint16_t*)out, y, gate_in, ldg, w, n, groups, eps);
    LAUNCH_OK(); return 0;
}

}  // extern "C"
