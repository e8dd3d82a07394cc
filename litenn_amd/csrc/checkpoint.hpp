// Host side: a JSON reader for model configurations and the safetensors container (an 8-byte
// little-endian header length, that many bytes of JSON mapping tensor names to dtype, shape and byte
// range, then the data).  The container is mapped read-only and every range is checked against the
// file before it is handed out.
#pragma once

#include <cstdint>
#include <map>
#include <memory>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

namespace litenn_hip
{
	class Json
	{
	public:
		enum Kind { Null, Bool, Number, String, Array, Object };
		Kind kind = Null;
		bool boolean = false;
		double number = 0.0;
		std::string text;
		std::vector<Json> items;
		std::vector<std::pair<std::string, Json>> members;

		// throws std::runtime_error naming `what` on malformed text
		static Json parse(const char* begin, size_t size, const std::string& what);

		const Json* find(const std::string& key) const;
		bool is_null() const { return kind == Null; }
		// the member's value; throws naming the key when it is absent or of another kind
		const Json& at(const std::string& key) const;
		double real(const std::string& key) const;
		// a whole number in [low, high]
		int integer(const std::string& key, int low, int high) const;
		const std::string& string(const std::string& key) const;
	};

	struct CheckpointTensor
	{
		std::string dtype;
		std::vector<size_t> shape;
		const uint8_t* data = nullptr;
		size_t bytes = 0;
	};

	class Safetensors
	{
	public:
		explicit Safetensors(const std::string& path); // throws std::runtime_error
		~Safetensors();
		Safetensors(const Safetensors&) = delete;
		Safetensors& operator=(const Safetensors&) = delete;
		const std::map<std::string, CheckpointTensor>& tensors() const { return tensors_; }

	private:
		void* map_ = nullptr;
		size_t size_ = 0;
		std::map<std::string, CheckpointTensor> tensors_;
	};

	std::string read_text_file(const std::string& path); // throws std::runtime_error
} // namespace litenn_hip
