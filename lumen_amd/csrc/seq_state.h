// What one live sequence holds between steps, in one slab per model: blocks that must start at zero (recurrent
// matrices, convolution and token-shift inputs) in front, rolling key / value stores, whose rows are written before
// they are read, behind.  A model reserves its blocks once, commits, and gets pointers that stay put, so recorded
// steps can hold them; reset() makes the slab ready for another sequence.
#pragma once
#include "internal.h"

class SeqState {
  public:
    enum Kind { ZEROED = 0, ROLLING = 1 };
    // -> handle of a block of that many floats (16-byte aligned)
    int reserve(Kind kind, size_t floats) {
        blocks_.push_back({kind, total_[kind], floats});
        total_[kind] += (floats + 3) & ~(size_t)3;
        return (int)blocks_.size() - 1;
    }
    int commit(lumen_ctx *ctx) {
        ctx_ = ctx;
        HIP_TRY(hipMalloc((void **)&slab_, (total_[0] + total_[1] + 4) * sizeof(float)));
        // (rolling stores once: rows are padded, and the padding is never written again)
        HIP_TRY(hipMemsetAsync(slab_, 0, (total_[0] + total_[1] + 4) * sizeof(float), ctx->stream));
        return LUMEN_OK;
    }
    int reset() {
        if (total_[0]) HIP_TRY(hipMemsetAsync(slab_, 0, total_[0] * sizeof(float), ctx_->stream));
        return LUMEN_OK;
    }
    float *ptr(int block) const { return slab_ + blocks_[block].offset + (blocks_[block].kind == ROLLING ? total_[0] : 0); }
    size_t floats(int block) const { return blocks_[block].floats; }
    size_t bytes() const { return (total_[0] + total_[1]) * sizeof(float); }
    ~SeqState() { hipFree(slab_); }

  private:
    struct Block {
        Kind kind;
        size_t offset, floats;
    };
    lumen_ctx *ctx_ = nullptr;
    float *slab_ = nullptr;
    size_t total_[2] = {0, 0};
    std::vector<Block> blocks_;
};
